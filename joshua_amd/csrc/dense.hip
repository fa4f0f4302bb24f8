// Products with plain weight rows and the mixture-of-experts backend on them (declared in dense.hpp).
#include "dense.hpp"

namespace jqh {

#define JQ_ELEM(TYPE, CALL)                                    \
    do {                                                       \
        if ((TYPE) == JQ_TYPE_BF16) {                          \
            using E = jq::ElemBf16;                            \
            CALL;                                              \
        } else {                                               \
            using E = jq::ElemF32;                             \
            CALL;                                              \
        }                                                      \
    } while (0)

namespace {

// The one-row product with the norm in front: a workgroup a compute unit, or a pair of rows a workgroup where there are
// fewer pairs.
template <bool GATED>
int run_norm_gemv(const jq_weight *w, const jq_weight *up, float *Y, const jq::GatedUnit &unit, const jq::ResidualNorm &nm, hipStream_t s) {
    const int k = (int)w->k, n = (int)w->n;
    if (nm.width != k || k > FUSED_NORM_MAX_WIDTH || nm.x_out == nm.x) return fail("dense gemv: no fused norm for this row");
    const uint8_t *wu = up ? up->dev : nullptr;
    const dim3 grid((unsigned)std::min(GATED ? n : (n + 1) / 2, 256));
#define JQ_NG(WAVES, NV)                                                                                                             \
    JQ_ELEM(w->type, hipLaunchKernelGGL((jq::norm_gemv<E, WAVES, NV, GATED>), grid, dim3(64 * WAVES), (size_t)k * sizeof(float), s, w->dev, \
                                        wu, w->row_bytes, Y, k, n, unit, nm))
    const bool few = (size_t)n * k <= ((size_t)1 << 20);  // a router, say: the norm is most of it
    if (few && k <= 1024) JQ_NG(4, 4);
    else if (few && k <= 4096) JQ_NG(4, 16);
    else if (k <= 2048) JQ_NG(8, 4);
    else if (k <= 4096) JQ_NG(16, 4);
    else JQ_NG(16, 8);
#undef JQ_NG
    note_kernel("norm_gemv");
    HIP_TRY(hipGetLastError());
    return 0;
}

}  // namespace

int dense_gemv(const jq_weight *w, const float *X, size_t ldx, int T, float *Y, size_t ldy, hipStream_t s, const jq::ResidualNorm *nm) {
    const int k = (int)w->k, n = (int)w->n;
    const dim3 grid((unsigned)((n + 3) / 4));
    if (T < 1 || T > GEMV_MAX_ROWS || (nm && T != 1)) return fail("dense gemv: %d rows", T);
    if (nm) return run_norm_gemv<false>(w, nullptr, Y, jq::GatedUnit{}, *nm, s);
    note_kernel("dense_gemv");
#define JQ_GEMV(MT)                                                                                                        \
    JQ_ELEM(w->type, hipLaunchKernelGGL((jq::dense_gemv<E, MT>), grid, dim3(256), 0, s, w->dev, w->row_bytes, X, ldx, Y, ldy, T, k, n))
    if (T == 1) JQ_GEMV(1);
    else if (T == 2) JQ_GEMV(2);
    else if (T <= 4) JQ_GEMV(4);
    else JQ_GEMV(8);
#undef JQ_GEMV
    HIP_TRY(hipGetLastError());
    return 0;
}

int dense_gemv_gated(const jq_weight *gate, const jq_weight *up, const float *X, size_t ldx, int T, float *Y, size_t ldy,
                     const jq::GatedUnit &unit, hipStream_t s, const jq::ResidualNorm *nm) {
    const int k = (int)gate->k, n = (int)gate->n;
    const dim3 grid((unsigned)((n + 1) / 2));
    if (T < 1 || T > GEMV_MAX_ROWS || (nm && T != 1)) return fail("dense gemv: %d rows", T);
    if (gate->type != up->type || up->n != gate->n || up->k != gate->k) return fail("dense gemv: gate and up differ");
    if (nm) return run_norm_gemv<true>(gate, up, Y, unit, *nm, s);
#define JQ_GEMV(MT)                                                                                                              \
    JQ_ELEM(gate->type, hipLaunchKernelGGL((jq::dense_gemv_gated<E, MT>), grid, dim3(256), 0, s, gate->dev, up->dev, gate->row_bytes, X, \
                                           ldx, Y, ldy, T, k, n, unit))
    if (T == 1) JQ_GEMV(1);
    else if (T == 2) JQ_GEMV(2);
    else if (T <= 4) JQ_GEMV(4);
    else JQ_GEMV(8);
#undef JQ_GEMV
    HIP_TRY(hipGetLastError());
    return 0;
}

namespace {

// How many runs a product's k is split into: one workgroup a tile fills the 256 compute units only from 256 tiles
// on.  Runs of at least 4 stages (512 bytes of a row); depends on the shape only, so a shape keeps its order of
// additions.
int gemm_splits(size_t tiles, int stages) {
    if (tiles >= 192) return tiles < 384 && stages >= 96 ? 2 : 1;  // long rows: a second workgroup a compute unit pays for the addition
    return (int)std::max<size_t>(1, std::min<size_t>({512 / tiles, (size_t)stages / 4, 16}));
}

template <class E, int BM, int BN, bool GATED, bool GROUPED>
void launch_gemm(const jq::DenseGemm &a, unsigned n_tiles, hipStream_t s) {
    hipLaunchKernelGGL((jq::dense_gemm<E, BM, BN, GATED, GROUPED>), dim3((unsigned)a.m_tiles * n_tiles, (unsigned)a.splits), dim3(256), 0, s, a);
}

// Tile of a product of `rows` activation rows (per group) and `wrows` weight rows: 128 x 128 where that makes enough
// tiles or the row count wants it, else smaller.
template <bool GATED, bool GROUPED>
int run_gemm(uint32_t type, jq::DenseGemm a, size_t rows_of_a, size_t k, size_t row_pairs, hipStream_t s) {
    const size_t esz = dense_elem_bytes(type);
    const size_t wrows = GATED ? 2 * (size_t)a.N : (size_t)a.N;
    if ((uint64_t)rows_of_a * a.lda >= (1ull << 32) || (uint64_t)a.N * a.ldw >= (1ull << 32))
        return fail("dense gemm: an operand of 4 GB or more");
    a.stages = (int)((k * esz + 127) / 128);
    auto tiles = [&](int bm, int bn) {
        const size_t mt = GROUPED ? (size_t)a.M / bm + a.groups : ((size_t)a.M + bm - 1) / bm;
        return std::make_pair(mt, (wrows + bn - 1) / bn);
    };
    int bm = 64, bn = 64;
    if (type == JQ_TYPE_BF16) {
        const size_t typical = GROUPED ? row_pairs : (size_t)a.M;  // rows a group has
        bm = typical > 96 ? 128 : 64, bn = 128;
        const auto t = tiles(bm, bn);
        if (t.first * t.second < 256 && bm == 128) bm = 64;
        const auto u = tiles(bm, bn);
        if (u.first * u.second < 128) bn = 64;
    }
    const auto t = tiles(bm, bn);
    if (t.first * t.second > 0x7FFFFFFFull) return fail("dense gemm: too many tiles");
    a.m_tiles = (int)t.first;
    a.splits = GROUPED || a.heads ? 1 : gemm_splits(t.first * t.second, a.stages);
    CallScratch scratch;
    float *C = a.C;
    if (a.splits > 1) {
        const size_t width = jq::gemm_partial_width(a.N, GATED);
        if (tl_fixed_scratch) {  // what a fixed scratch holds decides
            const size_t fit = tl_fixed_scratch->bytes / ((size_t)a.M * width * sizeof(float));
            a.splits = (int)std::min<size_t>((size_t)a.splits, std::max<size_t>(fit, 1));
        }
        uint8_t *p = nullptr;
        if (a.splits > 1) {
            if (scratch.get((size_t)a.splits * a.M * width * sizeof(float), s, &p)) return 1;
            a.C = (float *)p;
        }
    }
    if (type == JQ_TYPE_BF16) {
        if (bm == 128) launch_gemm<jq::ElemBf16, 128, 128, GATED, GROUPED>(a, (unsigned)t.second, s);
        else if (bn == 128) launch_gemm<jq::ElemBf16, 64, 128, GATED, GROUPED>(a, (unsigned)t.second, s);
        else launch_gemm<jq::ElemBf16, 64, 64, GATED, GROUPED>(a, (unsigned)t.second, s);
    } else {
        launch_gemm<jq::ElemF32, 64, 64, GATED, GROUPED>(a, (unsigned)t.second, s);
    }
    note_kernel(a.splits > 1 ? "dense_gemm+splitk" : "dense_gemm");
    if (a.splits > 1) {
        const size_t total = (size_t)a.M * a.N;
        if (GATED)
            JQ_ELEM(type, hipLaunchKernelGGL((jq::gemm_sum_splits_gated<E>), dim3(grid_for(total)), dim3(256), 0, s, a.C, a.splits,
                                             (size_t)a.M, a.N, (typename E::T *)a.act, a.ld_act, a.unit));
        else
            hipLaunchKernelGGL(jq::gemm_sum_splits, dim3(grid_for(total)), dim3(256), 0, s, a.C, a.splits, (size_t)a.M, a.N, C, a.ldc);
    }
    HIP_TRY(hipGetLastError());
    return 0;
}

}  // namespace

int dense_gemm(const jq_weight *w, const void *A, size_t lda, int T, float *C, size_t ldc, hipStream_t s) {
    if (lda < dense_stride(w->k) || lda % DENSE_PAD) return fail("dense gemm: activation rows of %zu elements for k = %zu", lda, w->k);
    jq::DenseGemm a{};
    a.A = (const uint8_t *)A, a.W = w->dev, a.lda = (uint32_t)(lda * dense_elem_bytes(w->type)), a.ldw = (uint32_t)w->row_bytes;
    a.M = T, a.N = (int)w->n, a.C = C, a.ldc = ldc;
    return run_gemm<false, false>(w->type, a, (size_t)T, w->k, 0, s);
}

int dense_gemm_heads(const jq_weight *w, size_t w_row, size_t n, const void *A, size_t lda, int T, void *out, int head_w, size_t head_stride,
                     size_t head_row, hipStream_t s) {
    if (lda < dense_stride(w->k) || lda % DENSE_PAD) return fail("dense gemm: activation rows of %zu elements for k = %zu", lda, w->k);
    if (head_w <= 0 || head_w % 4 || n % head_w || head_stride % 4 || head_row % 4 || w_row + n > w->n)
        return fail("dense gemm: %zu columns by heads of %d", n, head_w);
    jq::DenseGemm a{};
    a.A = (const uint8_t *)A, a.W = w->dev + w_row * w->row_bytes, a.lda = (uint32_t)(lda * dense_elem_bytes(w->type)), a.ldw = (uint32_t)w->row_bytes;
    a.M = T, a.N = (int)n, a.heads = out, a.head_w = head_w, a.head_stride = head_stride, a.head_row = head_row;
    return run_gemm<false, false>(w->type, a, (size_t)T, w->k, 0, s);
}

int dense_gemm_gated(const jq_weight *gate, const jq_weight *up, const void *A, size_t lda, int T, void *act, size_t ld_act,
                     const jq::GatedUnit &unit, hipStream_t s) {
    if (lda != dense_stride(gate->k)) return fail("dense gemm: activation rows of %zu elements for k = %zu", lda, gate->k);
    if (gate->type != up->type || up->n != gate->n || up->k != gate->k) return fail("dense gemm: gate and up differ");
    jq::DenseGemm a{};
    a.A = (const uint8_t *)A, a.W = gate->dev, a.W2 = up->dev, a.lda = (uint32_t)(lda * dense_elem_bytes(gate->type));
    a.ldw = (uint32_t)gate->row_bytes, a.M = T, a.N = (int)gate->n, a.act = act, a.ld_act = ld_act, a.unit = unit;
    return run_gemm<true, false>(gate->type, a, (size_t)T, gate->k, 0, s);
}

int rows_to_elem(uint32_t type, const float *X, size_t ldx, size_t rows, int k, void *out, size_t stride, hipStream_t s) {
    JQ_ELEM(type, hipLaunchKernelGGL((jq::rows_to_elem<E>), dim3(grid_for(rows * stride)), dim3(256), 0, s, X, ldx, rows, k,
                                     (typename E::T *)out, stride));
    HIP_TRY(hipGetLastError());
    return 0;
}

int dense_matmul(uint32_t type, const uint8_t *W, size_t row_bytes, const float *X, float *Y, size_t m, size_t k, size_t n,
                 hipStream_t s) {
    const jq_weight w{type, n, k, 0, row_bytes, const_cast<uint8_t *>(W), false};
    if (m <= (size_t)GEMV_MAX_ROWS) return dense_gemv(&w, X, k, (int)m, Y, n, s);
    const size_t stride = dense_stride(k), bytes = m * stride * dense_elem_bytes(type);
    // (the partial sums of a split product take the stream's other buffer)
    if (tl_fixed_scratch) {  // one array for everything: eight rows at a time, which need none
        for (size_t r = 0; r < m; r += GEMV_MAX_ROWS)
            if (dense_gemv(&w, X + r * k, k, (int)std::min<size_t>(GEMV_MAX_ROWS, m - r), Y + r * n, n, s)) return 1;
        return 0;
    }
    CallScratch scratch(1);
    uint8_t *acts = nullptr;
    if (scratch.get(bytes, s, &acts)) return 1;
    if (rows_to_elem(type, X, k, m, (int)k, acts, stride, s)) return 1;
    return dense_gemm(&w, acts, stride, (int)m, Y, n, s);
}

int dense_decode(const jq_weight *w, const uint32_t *ids, float *out, size_t rows, float scale, hipStream_t s) {
    if (!rows || !w->k) return 0;
    JQ_ELEM(w->type, hipLaunchKernelGGL((jq::dense_rows_to_f32<E>), dim3((unsigned)std::min<size_t>(rows, 65536), (unsigned)std::min<size_t>((w->k + 1023) / 1024, 64)), dim3(256), 0, s, w->dev, w->row_bytes, ids,
                                        out, rows, (int)w->k, scale));
    HIP_TRY(hipGetLastError());
    return 0;
}

int zero_floats(float *p, size_t n, hipStream_t s) {
    if (!n) return 0;
    hipLaunchKernelGGL(jq::fill_zero, dim3(grid_for(n)), dim3(256), 0, s, p, n);
    HIP_TRY(hipGetLastError());
    return 0;
}

int residual_norm(const jq::ResidualNorm &a, uint32_t type, void *he, size_t stride, size_t rows, const uint32_t *at, hipStream_t s) {
    if (a.width > NORM_MAX_WIDTH) return fail("residual norm: rows of %d exceed %d", a.width, NORM_MAX_WIDTH);
    if (!rows) return 0;
#define JQ_ROWS(NV, BT)                                                                                                          \
    JQ_ELEM(type, hipLaunchKernelGGL((jq::residual_norm_rows<E, NV, BT>), dim3((unsigned)rows), dim3(BT), 0, s, a, (typename E::T *)he, \
                                     stride, at))
    if (a.width <= 1024) JQ_ROWS(4, 256);
    else if (a.width <= 2048) JQ_ROWS(8, 256);
    else if (a.width <= 4096) JQ_ROWS(16, 256);
    else if (a.width <= 8192) JQ_ROWS(16, 512);
    else JQ_ROWS(16, 1024);
#undef JQ_ROWS
    HIP_TRY(hipGetLastError());
    return 0;
}

// ---- mixture of experts -----------------------------------------------------------------------------

namespace {

bool takes_dense(const jq_weight *gate, const jq_weight *up, const jq_weight *down) {
    return dense_elem_bytes(gate->type) && up->type == gate->type && down->type == gate->type;  // (a shared expert's: jq_moe_create)
}

int reserve_dense(jq_moe *m, size_t T) {
    const jq_moe_config &c = m->cfg;
    const size_t esz = dense_elem_bytes(m->gate->type), P = T * c.n_expert_used;
    HIP_TRY(hipMalloc((void **)&m->dense_x, T * dense_stride(c.hidden) * esz));
    HIP_TRY(hipMalloc((void **)&m->dense_act, P * dense_stride(c.inter) * esz));
    // (the columns behind inter stay zero: the kernels write the first inter only)
    HIP_TRY(hipMemset(m->dense_act, 0, P * dense_stride(c.inter) * esz));
    if (m->sgate) {
        const size_t bytes = T * dense_stride(m->sgate->n) * esz;
        HIP_TRY(hipMalloc((void **)&m->dense_sact, bytes));
        HIP_TRY(hipMemset(m->dense_sact, 0, bytes));
    }
    return 0;
}

void release_dense(jq_moe *m) {
    for (uint8_t *p : {m->dense_x, m->dense_act, m->dense_sact})
        if (p) (void)hipFree(p);
    m->dense_x = m->dense_act = m->dense_sact = nullptr;
}

// One expert is read by every pair that names it on the decode-sized kernels, once a row tile on the grouped GEMM.
bool decode_sized(const jq_moe_config &c, size_t T) { return T <= (size_t)GEMV_MAX_ROWS && T * c.n_expert_used <= 2 * (size_t)c.n_expert; }

}  // namespace

bool moe_dense_decode_sized(const jq_moe *m, size_t T) { return decode_sized(m->cfg, T); }

bool moe_dense_fuses_norm(const jq_moe *m, size_t T) {
    return T == 1 && m->cfg.hidden <= (uint32_t)FUSED_NORM_MAX_WIDTH && decode_sized(m->cfg, T);
}

int moe_forward_dense(jq_moe *m, size_t T, const float *x, const void *xe, float *y, hipStream_t s, const MoeDenseExtras &ex) {
    const jq_moe_config &c = m->cfg;
    const uint32_t type = m->gate->type;
    const int P = (int)(T * c.n_expert_used), h = (int)c.hidden, inter = (int)c.inter, ku = (int)c.n_expert_used;
    const jq::GatedUnit unit{c.swiglu_clamp > 0.0f ? c.swiglu_clamp : INFINITY, c.act_alpha == 0.0f ? 1.0f : c.act_alpha, c.act_up_shift};
    const jq::GatedUnit shared_unit{c.swiglu_clamp_shared > 0.0f ? c.swiglu_clamp_shared : INFINITY, unit.alpha, unit.shift};
    const jq::MoePairGroups no_groups{nullptr, nullptr, nullptr, nullptr, 0};
    const bool decode = decode_sized(c, T);
    const int sn = m->sgate ? (int)m->sgate->n : 0;
    if (m->sgate && (m->sgate->type != type || m->sup->type != type || m->sdown->type != type))
        return fail("moe: a shared expert of another type than the routed ones");
    // the shared expert's gate
    const float *sl = ex.logits ? ex.shared_logit : nullptr;
    size_t ld_sl = ex.ld;
    if (sn && m->sgate_row && !ex.logits) {
        if (ex.pre) return fail("moe: no fused norm in front of a gated shared expert");
        for (size_t t = 0; t < T; t += GEMV_MAX_ROWS)
            if (dense_gemv(m->sgate_row, x + t * h, h, (int)std::min<size_t>(GEMV_MAX_ROWS, T - t), m->sgate_logit + t, 1, s)) return 1;
        sl = m->sgate_logit, ld_sl = 1;
    }
    // the gating over logits that are there already, as a launch of its own
    jq::MoeGateParams gp = moe_gate_params(c);
    gp.ld = ex.logits ? (int)ex.ld : 0;
    auto gate = [&] { return moe_gate_dev(m, T, ex.logits ? ex.logits : m->logits, gp, no_groups, s); };
    if (decode) {
        const bool wave = moe_wave_gate(c);
        jq::MoeGateIn gi{ex.logits ? ex.logits : m->logits, m->router_bias, gp, m->ids, m->wts, no_groups, (int)T};
        if (ex.logits) {
            if (!wave && gate()) return 1;
        } else if (ex.pre) {  // residual update, norm and router logits in one launch; x is what it leaves
            const jq_weight packed{JQ_TYPE_F32, c.n_expert, c.hidden, 0, c.hidden * sizeof(float), (uint8_t *)m->router_w, false};
            const jq_weight &router = m->router_rows ? *m->router_rows : packed;
            if (ex.pre->h_out != x || T != 1) return fail("moe: the fused norm makes another row");
            if (dense_gemv(&router, nullptr, 0, 1, m->logits, c.n_expert, s, ex.pre)) return 1;
            if (!wave && gate()) return 1;
        } else {
            jq::MoeGateIn later{};
            if (moe_route_dev(m, T, x, s, no_groups, jq::ActsI8{nullptr, nullptr, nullptr, nullptr}, nullptr, wave ? &later : nullptr)) return 1;
        }
        const jq::SharedRows sh{sn ? m->sgate->dev : nullptr, sn ? m->sup->dev : nullptr, sn, m->sG, sl, ld_sl, P, shared_unit.limit};
        const dim3 grid((unsigned)((std::max(inter, sn) + 3) / 4), (unsigned)(P + (sn ? (int)T : 0)));
#define JQ_GU(NE)                                                                                                             \
    JQ_ELEM(type, hipLaunchKernelGGL((jq::moe_dense_gate_up<E, NE>), grid, dim3(256), 0, s, m->pgate, m->pup, m->gate->row_bytes, x, \
                                     (size_t)h, m->G, (size_t)inter, h, inter, ku, m->ids, unit, gi, sh))
        const int ne = (int)(c.n_expert + 63) / 64;
        if (!wave) JQ_GU(0);
        else if (ne == 1) JQ_GU(1);
        else if (ne == 2) JQ_GU(2);
        else if (ne == 3) JQ_GU(3);
        else JQ_GU(4);
#undef JQ_GU
        jq::SumRun shared_run{}, extra{};
        if (sn) shared_run = jq::SumRun{m->sdown->dev, m->sdown->row_bytes, m->sG, (size_t)sn, sn};
        if (ex.W) {
            if (T != 1 || ex.W->type != type || ex.W->n != c.hidden) return fail("moe: a product that does not join this result");
            extra = jq::SumRun{ex.W->dev, ex.W->row_bytes, ex.mid, ex.W->k, (int)ex.W->k};
        }
        JQ_ELEM(type, hipLaunchKernelGGL((jq::moe_dense_down<E>), dim3((unsigned)((h + 3) / 4), (unsigned)T), dim3(256), 0, s, m->pdown,
                                         m->down->row_bytes, m->G, (size_t)inter, m->ids, m->wts, y, inter, h, ku, (int)c.n_expert, shared_run,
                                         extra, ex.add));
        HIP_TRY(hipGetLastError());
        return 0;
    }
    if (ex.pre || ex.W) return fail("moe: no fused norm or product for %zu tokens", T);
    const size_t sx = dense_stride(c.hidden), sa = dense_stride(c.inter);
    if (!xe) {
        if (rows_to_elem(type, x, c.hidden, T, h, m->dense_x, sx, s)) return 1;
        xe = m->dense_x;
    }
    if ((ex.logits ? gate() : moe_route_dev(m, T, x, s, no_groups)) || moe_group_dev(m, T, 0, s)) return 1;
    const size_t esz = dense_elem_bytes(type), typical = ((size_t)P + c.n_expert - 1) / c.n_expert;
    jq::DenseGemm a{};
    a.A = (const uint8_t *)xe, a.Wp = m->pgate, a.Wp2 = m->pup, a.lda = (uint32_t)(sx * esz), a.ldw = (uint32_t)m->gate->row_bytes;
    a.M = P, a.N = inter, a.act = m->dense_act, a.ld_act = sa, a.unit = unit;
    a.offsets = m->offsets, a.xsel = m->xrow, a.groups = (int)c.n_expert;
    if (run_gemm<true, true>(type, a, T, c.hidden, typical, s)) return 1;
    jq::DenseGemm d{};
    d.A = m->dense_act, d.Wp = m->pdown, d.lda = (uint32_t)(sa * esz), d.ldw = (uint32_t)m->down->row_bytes;
    d.M = P, d.N = h, d.C = m->out, d.ldc = (size_t)h;
    d.offsets = m->offsets, d.yrow = m->yrow, d.groups = (int)c.n_expert;
    if (run_gemm<false, true>(type, d, (size_t)P, c.inter, typical, s)) return 1;
    if (sn && (dense_gemm_gated(m->sgate, m->sup, xe, sx, (int)T, m->dense_sact, dense_stride(sn), shared_unit, s) ||
               dense_gemm(m->sdown, m->dense_sact, dense_stride(sn), (int)T, m->sOut, h, s)))
        return 1;
    hipLaunchKernelGGL(jq::moe_combine_shared, dim3((unsigned)std::min<size_t>((T * h + 255) / 256, 4096)), dim3(256), 0, s, m->out, m->wts,
                       (int)T, ku, h, sn ? m->sOut : nullptr, sl, ld_sl, ex.add, y);
    HIP_TRY(hipGetLastError());
    return 0;
}

namespace {

int forward_dense(jq_moe *m, size_t T, const float *x, float *y, hipStream_t s, MoePreNorm *pre) {
    if (pre) return fail("moe: experts in plain rows take their norm as a launch of its own here");
    return moe_forward_dense(m, T, x, nullptr, y, s);
}

const MoeBackend g_dense_moe{takes_dense, reserve_dense, release_dense, forward_dense};
const RegisterMoeBackend g_register_dense_moe(&g_dense_moe);

}  // namespace

}  // namespace jqh
