// Layered decoders with plain BF16 / F32 weights: a stack whose layers each name a mixer (attention, selective scan,
// latent attention, matrix memory, linear attention with a constant decay) and a feed-forward block (none, dense, mixture
// of experts).  Mixer and block run one behind the other, each normalised in front and behind, or side by side on one
// norm; a run of layers may repeat.  A design is a reader of its configuration into StackConfig plus its tensor names;
// the step below runs any of them.
#include "dense.hpp"
#include "kernels_latent.hpp"
#include "kernels_linear.hpp"
#include "model.hpp"
#include "safetensors.hpp"

namespace {

// ---- what a design's configuration comes down to ------------------------------------------------------

struct RotaryConfig {
    int dims = 0;
    double base = 10000.0;
    double factor = 1.0, original = 0.0, fast = 0.0, slow = 0.0;  // YaRN; factor 1 with `yarn` false: none
    bool yarn = false;
    bool operator==(const RotaryConfig &o) const {
        return dims == o.dims && base == o.base && yarn == o.yarn && factor == o.factor && original == o.original && fast == o.fast && slow == o.slow;
    }
};

struct LayerConfig {
    enum Mixer { ATTENTION, MAMBA1, LATENT, MLSTM, LIGHTNING } mixer = ATTENTION;
    // attention of every kind
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    float scale = 1.0f;
    bool v_mix = false;
    RotaryConfig rot;
    int q_rank = 0, kv_rank = 0, rot_dim = 0;  // latent attention
    float gate_cap = 0.0f;                     // matrix memory
    std::vector<double> decay;                 // constant decay, one a head
    // selective scan
    int inner = 0, state = 0, dt_rank = 0, taps = 0;
    // feed-forward
    enum Mlp { NONE, DENSE, MOE } mlp = NONE;
    int ff = 0, experts = 0, top = 0, shared_ff = 0;
    float limit = INFINITY;

    bool linear() const { return mixer == MLSTM || mixer == LIGHTNING; }
    int state_rows() const { return vdim + (mixer == MLSTM ? 1 : 0); }  // of a head of a linear mixer
    int state_pitch() const { return (dim + 31) / 32 * 32; }
    int out_pitch() const { return (state_rows() + 3) / 4 * 4; }
    int latent_pitch() const { return (int)dense_stride(kv_rank + rot_dim); }
};

struct StackConfig {
    const char *arch = "";
    uint32_t vocab = 0, width = 0;
    float embedding_scale = 1.0f, norm_eps = 1e-6f, residual_mult = 1.0f;
    bool rms = false;                         // norms: root mean square instead of mean and variance with bias
    float act_alpha = 1.0f, act_shift = 0.0f;  // the gated unit: g sigmoid(alpha g) (u + shift)
    bool parallel = false;                    // x + (mixer(h) + block(h)) with h = norm1(x): one norm a layer
    int loop_start = 0, loop_stop = 0, loop_times = 1;  // layers start .. stop - 1 run that often in a row
    std::vector<LayerConfig> layers;
};

// The frequencies of the rotated pairs, and the factor on cos and sin.
double rotary_frequencies(const RotaryConfig &r, std::vector<double> *freq) {
    const int half = r.dims / 2;
    freq->resize(half);
    for (int i = 0; i < half; i++) (*freq)[i] = std::pow(r.base, -2.0 * i / r.dims);
    if (!r.yarn) return 1.0;
    // a pair keeps its frequency where it turns `fast` times or more over the original context, is slowed by
    // `factor` where it turns `slow` times or less, and goes over linearly between
    auto index_of = [&](double turns) { return r.dims * std::log(r.original / (2.0 * M_PI * turns)) / (2.0 * std::log(r.base)); };
    const double lo = std::max(std::floor(index_of(r.fast)), 0.0), hi = std::min(std::ceil(index_of(r.slow)), r.dims - 1.0);
    for (int i = 0; i < half; i++) {
        const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
        (*freq)[i] = (*freq)[i] / r.factor * ramp + (*freq)[i] * (1.0 - ramp);
    }
    return 0.1 * std::log(r.factor) + 1.0;
}

// ---- the model -----------------------------------------------------------------------------------------

struct NormWeights {
    float *w = nullptr, *b = nullptr;
};

struct Layer {
    LayerConfig c;
    NormWeights norm1, norm1b, norm2, norm2b;
    jq_weight *in = nullptr;   // q | k | v rows, or the scan's x | z
    jq_weight *o = nullptr;
    float lambda = 0.0f;
    bool v_first = false;      // the first layer that mixes values: the others mix in its own
    int rot = -1;              // which of the model's rotary tables
    // latent attention
    jq_weight *uq = nullptr, *ukv = nullptr;  // ukv: W_uk's rows, then W_uv's
    float *dq_norm = nullptr, *dkv_norm = nullptr, *sink = nullptr;
    // linear mixers
    float *i_b = nullptr, *f_b = nullptr, *decay = nullptr, *log_decay = nullptr;
    float *mix_norm = nullptr;
    // selective scan
    jq_weight *wx = nullptr, *wdt = nullptr;
    float *conv = nullptr, *conv_b = nullptr, *dt_b = nullptr, *A_log2 = nullptr, *D = nullptr;
    // places within a row of `in`'s product: the mixer's output gate, the router with the shared expert's gate behind it
    int gate_at = 0, router_at = 0;
    // feed-forward
    jq_weight *gate = nullptr, *up = nullptr, *down = nullptr;
    jq_moe *moe = nullptr;
    int moe_shares = -1;       // the first layer with experts of the same sizes: their scratch buffers take turns
    // this layer's activation buffers (shared between layers of equal size)
    void *mix_e = nullptr, *conv_e = nullptr, *dt_e = nullptr, *ff_e = nullptr;

    int DP() const { return (c.dim + c.rot_dim + 31) / 32 * 32; }
    int DVP() const { return (c.vdim + 31) / 32 * 32; }
    bool latent_by_heads() const { return c.dim % 4 == 0 && c.vdim % 4 == 0; }  // keys and values straight from the product
    int mix_width() const { return c.mixer == LayerConfig::MAMBA1 ? c.inner : c.heads * c.vdim; }
};

// One run of a layer within a step, with the cache or state that is its own.
struct LayerRun {
    int layer = 0;
    void *kc = nullptr, *vc = nullptr;  // attention; latent attention: kc holds the rows
    float *S = nullptr;                 // selective scan, linear mixers
    size_t S_floats = 0;
    float *tail[2] = {nullptr, nullptr};  // the scan's convolution, the matrix memory's running maxima: two taking turns
    size_t tail_floats = 0;
    int tail_at = 0;
};

struct RotaryTable {
    RotaryConfig c;
    double *freq = nullptr;
    float mag = 1.0f;
    float2 *cs = nullptr;  // [tokens of the step][dims / 2]
};

struct LayeredModel : jq_model {
    StackConfig cfg;
    uint32_t type = JQ_TYPE_BF16;  // of the matrices, the caches and a many-token step's activations
    std::vector<Layer> layers;
    std::vector<LayerRun> runs;
    std::vector<RotaryTable> rots;
    jq_weight *embed = nullptr, *head = nullptr;
    NormWeights final_norm;
    std::vector<void *> owned;     // weights and states in device memory
    std::vector<jq_weight *> matrices;
    // scratch for cap_tokens tokens, cap_want wanted rows and keys and values of cap_keys tokens out of latents
    size_t cap_tokens = 0, cap_want = 0, cap_keys = 0;
    std::vector<void *> scratch;
    uint32_t *ids = nullptr, *want_ids = nullptr;
    float *x = nullptr, *x2 = nullptr, *h = nullptr, *y = nullptr, *proj = nullptr, *mid = nullptr, *conv_f = nullptr, *bc = nullptr,
          *dt = nullptr, *first_v = nullptr, *part = nullptr, *lin_o = nullptr, *lin_m = nullptr, *cq = nullptr, *qf = nullptr,
          *qx = nullptr, *kv = nullptr, *lin_g = nullptr, *lin_S = nullptr;
    void *lin_e = nullptr, *h_e = nullptr, *q_e = nullptr, *cq_e = nullptr, *k_e = nullptr, *v_e = nullptr;
    std::vector<int> moe_holder;   // per layer index of the first of its size: which layer holds the scratch now
    bool broken = false;           // a step failed half way: the states are those of no sequence

    ~LayeredModel() override;
    int step(const uint32_t *tokens, uint32_t n, const uint32_t *want, uint32_t n_want, hipStream_t s) override;
    void forget() override { broken = false; }
    int reserve(size_t T, size_t W, size_t keys);
    int run_layers(int T, const uint32_t *want, int n_want, hipStream_t s);
    size_t esz() const { return dense_elem_bytes(type); }

    template <class T>
    int device_alloc(T **out, size_t n) {
        void *p = nullptr;
        HIP_TRY(hipMalloc(&p, std::max<size_t>(n * sizeof(T), 16)));
        owned.push_back(p);
        *out = (T *)p;
        return 0;
    }
};

void free_all(std::vector<void *> *v) {
    for (void *p : *v) (void)hipFree(p);
    v->clear();
}

LayeredModel::~LayeredModel() {
    for (Layer &l : layers) jq_moe_free(l.moe);
    for (jq_weight *w : matrices) jq_free(w);
    free_all(&scratch);
    free_all(&owned);
}

int LayeredModel::reserve(size_t T, size_t W, size_t keys) {
    if (T <= cap_tokens && W <= cap_want && keys <= cap_keys) return 0;
    T = std::max(T, cap_tokens), W = std::max(W, cap_want);
    keys = keys <= cap_keys ? cap_keys : std::min<size_t>(n_ctx, std::max(keys, 2 * cap_keys));  // (grows in few steps)
    free_all(&scratch);
    cap_tokens = cap_want = cap_keys = 0;
    size_t proj_w = 0, mid_w = 0, inner_w = 0, bc_w = 0, v_w = 0, part_w = 0, q_w = 0, lin_w = 0, head_w = 0, cq_w = 0, qf_w = 0, qx_w = 0,
           kv_w = 0, k_w = 0, ve_w = 0, lin_e_w = 0, lin_S_w = 0;
    const size_t seg = std::min<size_t>(T, jq::LIN_SEGMENT), chunks = (seg + jq::LIN_CHUNK - 1) / jq::LIN_CHUNK;
    for (const Layer &l : layers) {
        const LayerConfig &c = l.c;
        proj_w = std::max(proj_w, l.in->n);
        mid_w = std::max<size_t>({mid_w, (size_t)l.mix_width(), (size_t)c.ff});
        if (c.mixer == LayerConfig::ATTENTION) {
            q_w = std::max(q_w, (size_t)c.heads * l.DP());
            if (c.v_mix) v_w = std::max(v_w, (size_t)c.kv_heads * c.vdim);
            part_w = std::max(part_w, (size_t)c.heads * ((n_ctx + jq::ATT_CHUNK - 1) / jq::ATT_CHUNK) * (c.vdim + 2));
        } else if (c.mixer == LayerConfig::LATENT) {
            const size_t H = c.heads;
            q_w = std::max(q_w, H * l.DP()), cq_w = std::max(cq_w, (size_t)c.q_rank), qf_w = std::max(qf_w, l.uq->n);
            qx_w = std::max(qx_w, H * c.latent_pitch());
            part_w = std::max(part_w, H * jq::LAT_MAX_SPLIT * jq::latent_part_width(c.kv_rank));
            kv_w = std::max(kv_w, l.latent_by_heads() ? 0 : l.ukv->n), k_w = std::max(k_w, H * l.DP()), ve_w = std::max(ve_w, H * l.DVP());
        } else if (c.linear()) {
            lin_w = std::max(lin_w, (size_t)c.heads * c.out_pitch()), head_w = std::max(head_w, (size_t)c.heads);
            const size_t H = c.heads, rs = (c.state_rows() + 15) / 16 * 16;
            lin_e_w = std::max(lin_e_w, H * (2 * c.state_pitch() + rs)), lin_S_w = std::max(lin_S_w, H * rs * c.state_pitch());
        } else {
            inner_w = std::max(inner_w, (size_t)c.inner);
            bc_w = std::max(bc_w, l.wx->n);
        }
    }
    auto get = [&](auto **out, size_t n) {  // zeroed: the padding of activation rows is never written
        using P = std::remove_reference_t<decltype(**out)>;
        const size_t bytes = std::max<size_t>(n * sizeof(P), 256);
        void *p = nullptr;
        HIP_TRY(hipMalloc(&p, bytes));
        scratch.push_back(p);
        HIP_TRY(hipMemset(p, 0, bytes));
        *out = (P *)p;
        return 0;
    };
    const size_t w = cfg.width, R = std::max(T, W);
    if (get(&ids, T) || get(&want_ids, W) || get(&x, T * w) || get(&x2, w) || get(&h, R * w) || get(&y, T * w) || get(&proj, T * proj_w) ||
        get(&mid, (size_t)GEMV_MAX_ROWS * mid_w) || get(&conv_f, (size_t)GEMV_MAX_ROWS * inner_w) || get(&bc, T * bc_w) ||
        get(&dt, T * inner_w) || get(&first_v, T * v_w) || get(&part, (size_t)GEMV_MAX_ROWS * part_w) || get(&lin_o, T * lin_w) ||
        get(&lin_m, T * head_w) || get(&cq, (size_t)GEMV_MAX_ROWS * cq_w) || get(&qf, T * qf_w) || get(&qx, (size_t)GEMV_MAX_ROWS * qx_w) ||
        get(&kv, keys * kv_w))
        return 1;
    const bool chunked = type == JQ_TYPE_BF16 && T > (size_t)GEMV_MAX_ROWS;
    if (chunked && lin_S_w && (get(&lin_g, head_w * chunks * (2 * jq::LIN_CHUNK + 2)) || get(&lin_S, chunks * lin_S_w))) return 1;
    uint8_t *p = nullptr;
    if (get(&p, R * dense_stride(w) * esz())) return 1;
    h_e = p;
    if (get(&p, T * q_w * esz())) return 1;
    q_e = p;
    if (get(&p, T * dense_stride(cq_w) * esz())) return 1;
    cq_e = p;
    if (chunked && lin_S_w) {
        if (get(&p, seg * lin_e_w * esz())) return 1;
        lin_e = p;
    }
    if (get(&p, keys * k_w * esz())) return 1;
    k_e = p;
    if (get(&p, keys * ve_w * esz())) return 1;
    v_e = p;
    for (RotaryTable &r : rots)
        if (get(&r.cs, T * (r.c.dims / 2))) return 1;
    std::map<std::pair<int, size_t>, void *> by_size;  // (role, row length)
    auto rows = [&](int role, size_t k, void **out) {
        void *&slot = by_size[{role, k}];
        if (!slot) {
            uint8_t *b = nullptr;
            if (get(&b, T * dense_stride(k) * esz())) return 1;
            slot = b;
        }
        *out = slot;
        return 0;
    };
    for (Layer &l : layers) {
        if (rows(0, l.mix_width(), &l.mix_e)) return 1;
        if (l.c.mixer == LayerConfig::MAMBA1 && (rows(1, l.c.inner, &l.conv_e) || rows(2, l.c.dt_rank, &l.dt_e))) return 1;
        if (l.c.mlp == LayerConfig::DENSE && rows(3, l.c.ff, &l.ff_e)) return 1;
    }
    cap_tokens = T, cap_want = W, cap_keys = keys;
    return 0;
}

int LayeredModel::step(const uint32_t *tokens, uint32_t n, const uint32_t *want, uint32_t n_want, hipStream_t s) {
    if (broken) return fail("%s: an earlier step failed half way; reset the model", arch);
    bool latent = false;
    for (const Layer &l : layers) latent |= l.c.mixer == LayerConfig::LATENT;
    if (reserve(n, std::max<uint32_t>(n_want, 1), latent && n > (uint32_t)GEMV_MAX_ROWS ? n_past + n : 0)) return 1;
    HIP_TRY(hipMemcpyAsync(ids, tokens, n * sizeof(uint32_t), hipMemcpyHostToDevice, s));
    if (n_want && n > 1) HIP_TRY(hipMemcpyAsync(want_ids, want, n_want * sizeof(uint32_t), hipMemcpyHostToDevice, s));
    broken = true;
    if (run_layers((int)n, want, (int)n_want, s)) return 1;
    HIP_TRY(hipGetLastError());
    broken = false;
    return 0;
}

#define JQ_ELEM_OF(TYPE, CALL)                                 \
    do {                                                       \
        if ((TYPE) == JQ_TYPE_BF16) {                          \
            using E = jq::ElemBf16;                            \
            CALL;                                              \
        } else {                                               \
            using E = jq::ElemF32;                             \
            CALL;                                              \
        }                                                      \
    } while (0)

// Attention of the queries in q_e over the keys and values in a.kc and a.vc.
int run_attention_rows(LayeredModel *m, const jq::AttnLayer &a, bool small, float *out_f, void *out_e, hipStream_t s) {
    const uint32_t type = m->type;
    const int dk = a.DP, dv = a.DVP, gq = a.H / a.G, T = a.T;
    const size_t ldo = dense_stride((size_t)a.H * a.dv);
    if (type == JQ_TYPE_BF16 && dk <= 256 && dv <= 256 && !small && a.scale > 0.0f) {
        const float sl = a.scale * 1.44269504088896341f;
        const size_t rows = (size_t)T * gq;
        // two sets of 16 rows a wave where that still makes a workgroup for every compute unit
        const bool two = dk <= 192 && dv <= 128 && (rows + 127) / 128 * a.G >= 256;
        const dim3 grid((unsigned)((rows + (two ? 127 : 63)) / (two ? 128 : 64)), (unsigned)a.G);
        const __bf16 *q = (const __bf16 *)m->q_e;
        __bf16 *o = (__bf16 *)out_e;
#define JQ_TILES(DK, DV, QF, KT) hipLaunchKernelGGL((jq::attention_tiles_bf16<DK, DV, QF, KT>), grid, dim3(256), 0, s, a, q, o, ldo, sl)
        if (dk <= 64 && dv <= 64 && two) JQ_TILES(64, 64, 2, 64);
        else if (dk <= 64 && dv <= 64) JQ_TILES(64, 64, 1, 64);
        else if (dk <= 128 && dv <= 128 && two) JQ_TILES(128, 128, 2, 64);
        else if (dk <= 128 && dv <= 128) JQ_TILES(128, 128, 1, 64);
        else if (dk <= 192 && dv <= 128 && two) JQ_TILES(192, 128, 2, 64);
        else if (dk <= 192 && dv <= 128) JQ_TILES(192, 128, 1, 64);
        else JQ_TILES(256, 256, 1, 32);
#undef JQ_TILES
        return 0;
    }
    const size_t lds = ((size_t)a.DP + jq::ANY_CHUNK + 16 + 256) * sizeof(float);
    if (small)
        JQ_ELEM_OF(type, hipLaunchKernelGGL((jq::attention_any<E, float>), dim3((unsigned)(T * a.H)), dim3(256), lds, s, a,
                                            (const typename E::T *)m->q_e, out_f, (size_t)a.H * a.dv));
    else
        JQ_ELEM_OF(type, hipLaunchKernelGGL((jq::attention_any<E, typename E::T>), dim3((unsigned)(T * a.H)), dim3(256), lds, s, a,
                                            (const typename E::T *)m->q_e, (typename E::T *)out_e, ldo));
    return 0;
}

// The attention of one layer over its projections a.qkv.  Steps of up to 8 tokens leave f32 rows in out_f, longer
// ones rows of the element type in out_e.
int run_attention(LayeredModel *m, Layer &l, const jq::AttnLayer &a, bool small, float *out_f, void *out_e, hipStream_t s) {
    const uint32_t type = m->type;
    const int dc = std::max(a.DP, a.DVP), gq = a.H / a.G, T = a.T;
    if (small && dc <= 256) {
        const int n_chunks = (a.pos0 + T + jq::ATT_CHUNK - 1) / jq::ATT_CHUNK;
        // a query head a workgroup until there are four for every compute unit, then more
        const int per = std::min({gq, jq::DEC_HEADS, std::max(1, n_chunks * a.G * gq * T / 1024)}), runs = (gq + per - 1) / per;
        const dim3 grid((unsigned)((n_chunks * a.G + 7) / 8 * 8 * runs), (unsigned)T);
#define JQ_DEC(DC) JQ_ELEM_OF(type, hipLaunchKernelGGL((jq::attention_decode<E, DC>), grid, dim3(256), 0, s, a, n_chunks, per, m->part))
        if (dc <= 64) JQ_DEC(64);
        else if (dc <= 128) JQ_DEC(128);
        else JQ_DEC(256);
#undef JQ_DEC
        hipLaunchKernelGGL(jq::attention_merge, dim3((unsigned)(T * a.H)), dim3(128), 2 * n_chunks * sizeof(float), s, m->part, out_f, a.dv,
                           n_chunks);
        return 0;
    }
    JQ_ELEM_OF(type, hipLaunchKernelGGL((jq::attn_rope_store<E>), dim3((unsigned)T), dim3(256), 0, s, a, (typename E::T *)m->q_e));
    return run_attention_rows(m, a, small, out_f, out_e, s);
}

template <class IO>
int run_scan(const jq::SsmScan &a, const IO *x, IO *out, hipStream_t s) {
#define JQ_SCAN(LPC, NS)                                                                                                            \
    hipLaunchKernelGGL((jq::selective_scan<LPC, NS, IO>), dim3((unsigned)((a.C + 256 / LPC - 1) / (256 / LPC))), dim3(256), 0, s, a, x, out)
    if (a.N <= 4) JQ_SCAN(4, 1);
    else if (a.N <= 8) JQ_SCAN(4, 2);
    else if (a.N <= 16) JQ_SCAN(8, 2);
    else if (a.N <= 32) JQ_SCAN(16, 2);
    else if (a.N <= 64) JQ_SCAN(16, 4);
    else if (a.N <= 128) JQ_SCAN(32, 4);
    else if (a.N <= 256) JQ_SCAN(64, 4);
    else JQ_SCAN(64, 8);
#undef JQ_SCAN
    return 0;
}

// The linear mixers: kernels_linear.hpp over the projections, then the norm and gate of the heads' outputs.
int run_linear(LayeredModel *m, const Layer &l, LayerRun &r, int T, bool small, hipStream_t s) {
    const LayerConfig &c = l.c;
    jq::LinearLayer a{};
    a.H = c.heads, a.d = c.dim, a.dv = c.vdim, a.rows = c.state_rows(), a.DP = c.state_pitch(), a.memory = c.mixer == LayerConfig::MLSTM;
    a.T = T, a.proj = m->proj, a.ld = l.in->n, a.q_at = 0, a.k_at = c.heads * c.dim, a.v_at = 2 * a.k_at;
    a.i_at = l.gate_at + c.heads * c.vdim, a.f_at = a.i_at + c.heads;
    a.q_scale = a.memory ? 1.0f / std::sqrt((float)c.dim) : 1.0f, a.cap = c.gate_cap, a.i_b = l.i_b, a.f_b = l.f_b;
    a.decay = l.decay, a.log_decay = l.log_decay, a.S = r.S, a.m_in = r.tail[r.tail_at], a.m_out = r.tail[r.tail_at ^ 1];
    a.o = m->lin_o, a.OP = c.out_pitch(), a.mt = m->lin_m;
    if (m->type == JQ_TYPE_BF16 && !small) {
        jq::LinearChunks k{};
        k.H = a.H, k.DQ = a.DP, k.VP = k.RS = (a.rows + 15) / 16 * 16, k.OP = a.OP, k.S = m->lin_S;
        const unsigned H = (unsigned)a.H, row_runs = (unsigned)((k.RS + 63) / 64);
        for (int t0 = 0; t0 < T; t0 += jq::LIN_SEGMENT) {
            jq::LinearLayer b = a;
            b.T = std::min(jq::LIN_SEGMENT, T - t0), b.proj += (size_t)t0 * b.ld, b.o += (size_t)t0 * b.H * b.OP, b.mt += (size_t)t0 * b.H;
            b.m_in = r.tail[r.tail_at], b.m_out = r.tail[r.tail_at ^ 1];
            k.T = b.T, k.nc = (b.T + jq::LIN_CHUNK - 1) / jq::LIN_CHUNK, k.o = b.o;
            k.q = (__bf16 *)m->lin_e, k.k = k.q + (size_t)k.T * k.H * k.DQ, k.v = k.k + (size_t)k.T * k.H * k.DQ;
            const size_t places = (size_t)k.H * k.nc * jq::LIN_CHUNK;
            k.gi = m->lin_g, k.gf = k.gi + places, k.m_at = k.gf + places, k.carry = k.m_at + (size_t)k.H * k.nc;
            const dim3 grid((unsigned)k.nc, row_runs, H);
            hipLaunchKernelGGL(jq::linear_prepare, dim3((unsigned)k.T), dim3(256), 0, s, b, k);
            hipLaunchKernelGGL(jq::linear_gates, dim3(H), dim3(1024), 0, s, b, k);
            hipLaunchKernelGGL(jq::linear_chunk_state, grid, dim3(256), 0, s, k);
            hipLaunchKernelGGL(jq::linear_state_pass, dim3((unsigned)((a.rows * (k.DQ / 4) + 255) / 256), H), dim3(256), 0, s, k, r.S, a.rows);
            if (k.RS <= 64) hipLaunchKernelGGL((jq::linear_chunk_out<1>), grid, dim3(256), 0, s, k);
            else hipLaunchKernelGGL((jq::linear_chunk_out<2>), dim3((unsigned)k.nc, (unsigned)((k.RS + 127) / 128), H), dim3(256), 0, s, k);
            if (a.memory) r.tail_at ^= 1;
        }
    } else {
#define JQ_STEPS(LPR, NS)                                                                                                             \
    hipLaunchKernelGGL((jq::linear_steps<LPR, NS>), dim3((unsigned)((a.rows + 256 / LPR - 1) / (256 / LPR)), (unsigned)a.H), dim3(256), 0, s, a)
        if (a.d <= 16) JQ_STEPS(4, 1);
        else if (a.d <= 32) JQ_STEPS(8, 1);
        else if (a.d <= 64) JQ_STEPS(16, 1);
        else if (a.d <= 128) JQ_STEPS(16, 2);
        else if (a.d <= 256) JQ_STEPS(16, 4);
        else if (a.d <= 512) JQ_STEPS(32, 4);
        else JQ_STEPS(64, 4);
#undef JQ_STEPS
        if (a.memory) r.tail_at ^= 1;
    }
    jq::LinearNorm n{};
    n.o = m->lin_o, n.mt = m->lin_m, n.H = a.H, n.dv = a.dv, n.OP = a.OP, n.memory = n.per_head = a.memory, n.w = l.mix_norm;
    n.gate = m->proj + l.gate_at, n.ld = a.ld, n.eps = m->cfg.norm_eps;
    const int len = n.per_head ? a.dv : a.H * a.dv;
    const dim3 grid((unsigned)(n.per_head ? T * a.H : T));
#define JQ_NORM(BT)                                                                                                                    \
    do {                                                                                                                               \
        if (small) hipLaunchKernelGGL((jq::linear_norm_gate<float, BT>), grid, dim3(BT), 0, s, n, m->mid, (size_t)l.mix_width());       \
        else JQ_ELEM_OF(m->type, hipLaunchKernelGGL((jq::linear_norm_gate<typename E::T, BT>), grid, dim3(BT), 0, s, n,                 \
                                                    (typename E::T *)l.mix_e, dense_stride(l.mix_width())));                           \
    } while (0)
    if (len <= 256) JQ_NORM(64);
    else if (len <= 1024) JQ_NORM(256);
    else JQ_NORM(1024);
#undef JQ_NORM
    return 0;
}

int run_latent(LayeredModel *m, const Layer &l, const LayerRun &r, int pos0, int T, bool small, hipStream_t s) {
    const LayerConfig &c = l.c;
    const uint32_t type = m->type;
    const size_t sq = dense_stride(c.q_rank), ld = l.in->n;
    jq::LatentLayer a{};
    a.H = c.heads, a.d = c.dim, a.rd = c.rot_dim, a.dv = c.vdim, a.R = c.kv_rank, a.RP = c.latent_pitch(), a.n_ctx = (int)m->n_ctx;
    a.rot = c.rot.dims, a.pos0 = pos0, a.T = T, a.scale = c.scale, a.eps = m->cfg.norm_eps, a.q = m->qf, a.down = m->proj + c.q_rank, a.ld = ld;
    a.cs = l.rot >= 0 ? m->rots[l.rot].cs : nullptr, a.norm_w = l.dkv_norm, a.sink = l.sink, a.gate = m->proj + l.gate_at, a.cache = r.kc;
    // the queries, through their normed latent (the first numbers of a projection row)
    jq::ResidualNorm nm{};
    nm.x = m->proj, nm.ldx = ld, nm.pre_w = l.dq_norm, nm.eps = m->cfg.norm_eps, nm.rms = 1, nm.width = c.q_rank;
    if (T == 1 && c.q_rank <= FUSED_NORM_MAX_WIDTH) {
        if (dense_gemv(l.uq, nullptr, 0, 1, m->qf, l.uq->n, s, &nm)) return 1;
    } else if (small) {
        nm.h_out = m->cq;
        if (residual_norm(nm, type, nullptr, 0, T, nullptr, s) || dense_gemv(l.uq, m->cq, c.q_rank, T, m->qf, l.uq->n, s)) return 1;
    } else if (residual_norm(nm, type, m->cq_e, sq, T, nullptr, s) || dense_gemm(l.uq, m->cq_e, sq, T, m->qf, l.uq->n, s)) {
        return 1;
    }
    if (small) {
        const size_t pitch = l.ukv->row_bytes;
        const uint8_t *Wuk = l.ukv->dev, *Wuv = Wuk + (size_t)a.H * a.d * pitch;
        const unsigned H = (unsigned)a.H, Tu = (unsigned)T;
        const int n_split = std::min(jq::LAT_MAX_SPLIT, (pos0 + T + jq::LAT_RUN - 1) / jq::LAT_RUN);
        const dim3 absorb((unsigned)((a.R + 16 * (type == JQ_TYPE_BF16 ? jq::ElemBf16::CH : jq::ElemF32::CH) - 1) /
                                     (16 * (type == JQ_TYPE_BF16 ? jq::ElemBf16::CH : jq::ElemF32::CH))), H + 1, Tu);
        if (type == JQ_TYPE_BF16 && a.R <= 1024) {
            const dim3 grid((unsigned)n_split, (H + 15) / 16, Tu);
            __bf16 *qb = (__bf16 *)m->qx;
            hipLaunchKernelGGL((jq::latent_absorb<jq::ElemBf16, __bf16>), absorb, dim3(256), 0, s, a, Wuk, pitch, qb);
            if (a.R <= 256) hipLaunchKernelGGL((jq::latent_attention_mfma<1>), grid, dim3(256), 0, s, a, qb, n_split, m->part);
            else if (a.R <= 512) hipLaunchKernelGGL((jq::latent_attention_mfma<2>), grid, dim3(256), 0, s, a, qb, n_split, m->part);
            else hipLaunchKernelGGL((jq::latent_attention_mfma<4>), grid, dim3(256), 0, s, a, qb, n_split, m->part);
        } else {
            JQ_ELEM_OF(type, hipLaunchKernelGGL((jq::latent_absorb<E, float>), absorb, dim3(256), 0, s, a, Wuk, pitch, m->qx));
            JQ_ELEM_OF(type, hipLaunchKernelGGL((jq::latent_attention_any<E>), dim3((unsigned)n_split, H, Tu), dim3(256),
                                                (size_t)(a.RP + jq::LAT_RUN) * sizeof(float), s, a, m->qx, n_split, m->part));
        }
        const dim3 values((unsigned)((a.dv + 4 * jq::LAT_VROWS - 1) / (4 * jq::LAT_VROWS)), H, Tu);
#define JQ_VALUES(NS) JQ_ELEM_OF(type, hipLaunchKernelGGL((jq::latent_values<E, NS>), values, dim3(256), 0, s, a, m->part, n_split, Wuv, pitch, m->mid))
        if (n_split <= 16) JQ_VALUES(16);
        else JQ_VALUES(jq::LAT_MAX_SPLIT);
#undef JQ_VALUES
        return 0;
    }
    const int n = pos0 + T, DP = l.DP(), DVP = l.DVP();
    JQ_ELEM_OF(type, hipLaunchKernelGGL((jq::latent_store<E>), dim3((unsigned)T), dim3(256), 0, s, a));
    if (l.latent_by_heads()) {
        const size_t nk = (size_t)a.H * a.d, nv = (size_t)a.H * a.dv;
        if (dense_gemm_heads(l.ukv, 0, nk, r.kc, (size_t)a.RP, n, m->k_e, a.d, (size_t)n * DP, (size_t)DP, s) ||
            dense_gemm_heads(l.ukv, nk, nv, r.kc, (size_t)a.RP, n, m->v_e, a.dv, (size_t)n * DVP, (size_t)DVP, s))
            return 1;
        JQ_ELEM_OF(type, hipLaunchKernelGGL((jq::latent_rest_of_keys<E>), dim3((unsigned)n), dim3(256), 0, s, a, n, DP, DVP, (typename E::T *)m->k_e,
                                            (typename E::T *)m->v_e));
    } else {
        if (dense_gemm(l.ukv, r.kc, (size_t)a.RP, n, m->kv, l.ukv->n, s)) return 1;
        const unsigned gy = (unsigned)std::min((a.H * (DP + DVP) + 255) / 256, 16);
        JQ_ELEM_OF(type, hipLaunchKernelGGL((jq::latent_expand<E>), dim3((unsigned)n, gy), dim3(256), 0, s, a, m->kv, n, DP, DVP, (typename E::T *)m->k_e,
                                            (typename E::T *)m->v_e));
    }
    JQ_ELEM_OF(type, hipLaunchKernelGGL((jq::latent_queries<E>), dim3((unsigned)T), dim3(256), 0, s, a, DP, (typename E::T *)m->q_e));
    jq::AttnLayer t{};
    t.H = t.G = a.H, t.d = c.dim + c.rot_dim, t.dv = a.dv, t.DP = DP, t.DVP = DVP, t.n_ctx = n, t.scale = a.scale, t.pos0 = pos0, t.T = T;
    t.kc = m->k_e, t.vc = m->v_e, t.sink = a.sink, t.gate = a.gate, t.ld_gate = ld;
    return run_attention_rows(m, t, false, nullptr, l.mix_e, s);
}

int run_mamba(LayeredModel *m, const Layer &l, LayerRun &r, int T, bool small, hipStream_t s) {
    const LayerConfig &c = l.c;
    const uint32_t type = m->type;
    const int C = c.inner, N = c.state, taps = c.taps;
    const dim3 cgrid((unsigned)((C + 255) / 256), (unsigned)((T + taps - 1 + jq::CONV_RUN - 1) / jq::CONV_RUN));
    float *t_in = r.tail[r.tail_at], *t_out = r.tail[r.tail_at ^ 1];
    if (small)
        hipLaunchKernelGGL((jq::causal_conv_silu<float>), cgrid, dim3(256), 0, s, m->proj, l.in->n, l.conv, l.conv_b, t_in, t_out, m->conv_f, (size_t)C,
                           T, C, taps);
    else
        JQ_ELEM_OF(type, hipLaunchKernelGGL((jq::causal_conv_silu<typename E::T>), cgrid, dim3(256), 0, s, m->proj, l.in->n, l.conv, l.conv_b, t_in,
                                            t_out, (typename E::T *)l.conv_e, dense_stride(C), T, C, taps));
    r.tail_at ^= 1;
    const size_t ldp = l.wx->n;
    if (small ? dense_gemv(l.wx, m->conv_f, C, T, m->bc, ldp, s) : dense_gemm(l.wx, l.conv_e, dense_stride(C), T, m->bc, ldp, s)) return 1;
    jq::SsmScan a{};
    a.dt_raw = m->dt, a.dt_bias = l.dt_b, a.bc = m->bc + c.dt_rank, a.ld_bc = ldp, a.z = m->proj + C, a.ld_z = l.in->n;
    a.A_log2 = l.A_log2, a.D = l.D, a.S = r.S, a.T = T, a.C = C, a.N = N, a.ldx = a.ldo = (size_t)C;
    if (T == 1) {
        JQ_ELEM_OF(type, hipLaunchKernelGGL((jq::selective_step<E>), dim3((unsigned)((C + 15) / 16)), dim3(256), 0, s, a, l.wdt->dev, l.wdt->row_bytes,
                                            m->bc, c.dt_rank, m->conv_f, m->mid));
    } else if (small) {
        if (dense_gemv(l.wdt, m->bc, ldp, T, m->dt, C, s) || run_scan<float>(a, m->conv_f, m->mid, s)) return 1;
    } else {
        const size_t sr = dense_stride(c.dt_rank);
        if (rows_to_elem(type, m->bc, ldp, T, c.dt_rank, l.dt_e, sr, s) || dense_gemm(l.wdt, l.dt_e, sr, T, m->dt, C, s)) return 1;
        a.ldx = a.ldo = dense_stride(C);
        JQ_ELEM_OF(type, if (run_scan<typename E::T>(a, (const typename E::T *)l.conv_e, (typename E::T *)l.mix_e, s)) return 1);
    }
    return 0;
}

int LayeredModel::run_layers(int T, const uint32_t *want, int n_want, hipStream_t s) {
    const int w = (int)cfg.width;
    const size_t sw = dense_stride(w);
    const bool small = T <= GEMV_MAX_ROWS;             // f32 activations through the GEMV
    const bool one = T == 1 && w <= FUSED_NORM_MAX_WIDTH;  // and the residual update and norm inside the product's launch
    const int pos0 = (int)n_past;
    if (dense_decode(embed, ids, x, T, cfg.embedding_scale, s)) return 1;
    for (const RotaryTable &r : rots)
        hipLaunchKernelGGL(jq::rope_angles, dim3(grid_for((size_t)T * (r.c.dims / 2))), dim3(256), 0, s, r.freq, r.c.dims / 2, pos0, T, r.mag, r.cs);
    if (pos0 == 0) {  // a new sequence: its states start at zero
        for (LayerRun &r : runs)
            if (zero_floats(r.S, r.S_floats, s) || zero_floats(r.tail[r.tail_at], r.tail_floats, s)) return 1;
    }
    float *xc = x, *xo = x2;
    const float *pending = nullptr;       // the sublayer result not yet in the stream, and the norm it takes first
    NormWeights post;
    // the residual update with `pre` as the next norm; out: where the stream goes
    auto update = [&](const NormWeights &pre, float *out, float *h_out) {
        jq::ResidualNorm nm{};
        nm.x = xc, nm.y = pending, nm.post_w = post.w, nm.post_b = post.b, nm.mult = cfg.residual_mult;
        nm.pre_w = pre.w, nm.pre_b = pre.b, nm.eps = cfg.norm_eps, nm.rms = cfg.rms ? 1 : 0, nm.width = w;
        nm.x_out = out, nm.h_out = h_out;
        return nm;
    };
    // out [T][wt->n] = wt norm(stream), the stream updated on the way; `keep`: the normed rows stay, in h up to 8 tokens
    // and in h_e from there on
    auto norm_product = [&](const NormWeights &pre, const jq_weight *wt, float *out, bool keep) {
        if (one) {
            const jq::ResidualNorm nm = update(pre, xo, keep ? h : nullptr);
            if (dense_gemv(wt, nullptr, 0, 1, out, wt->n, s, &nm)) return 1;
            std::swap(xc, xo);
            return 0;
        }
        if (residual_norm(update(pre, xc, small ? h : nullptr), type, small ? nullptr : h_e, sw, T, nullptr, s)) return 1;
        return small ? dense_gemv(wt, h, w, T, out, wt->n, s) : dense_gemm(wt, h_e, sw, T, out, wt->n, s);
    };
    // the experts of a layer, their scratch handed over from the layer of their sizes that had it last
    auto experts = [&](Layer &l, const float *hx, const void *hxe, const MoeDenseExtras &ex) {
        int &holder = moe_holder[l.moe_shares];
        if (layers[holder].moe != l.moe) moe_swap_scratch(l.moe, layers[holder].moe);
        holder = (int)(&l - layers.data());
        std::lock_guard<std::mutex> lock(l.moe->mu);
        return moe_reserve(l.moe, cap_tokens) || moe_forward_dense(l.moe, T, hx, hxe, y, s, ex);
    };
    for (LayerRun &r : runs) {
        Layer &l = layers[r.layer];
        const LayerConfig &c = l.c;
        const bool beside = cfg.parallel && c.mlp != LayerConfig::NONE;
        if (norm_product(l.norm1, l.in, proj, beside)) return 1;
        switch (c.mixer) {
        case LayerConfig::ATTENTION: {
            jq::AttnLayer a{};
            a.H = c.heads, a.G = c.kv_heads, a.d = c.dim, a.dv = c.vdim, a.DP = l.DP(), a.DVP = l.DVP(), a.n_ctx = (int)n_ctx;
            a.rot = c.rot.dims, a.scale = c.scale, a.pos0 = pos0, a.T = T, a.qkv = proj, a.ld = l.in->n, a.cs = l.rot >= 0 ? rots[l.rot].cs : nullptr;
            a.v_first = c.v_mix && !l.v_first ? first_v : nullptr, a.v_first_out = l.v_first ? first_v : nullptr, a.lambda = l.lambda;
            a.kc = r.kc, a.vc = r.vc;
            if (run_attention(this, l, a, small, mid, l.mix_e, s)) return 1;
            break;
        }
        case LayerConfig::MAMBA1:
            if (run_mamba(this, l, r, T, small, s)) return 1;
            break;
        case LayerConfig::LATENT:
            if (run_latent(this, l, r, pos0, T, small, s)) return 1;
            break;
        default:
            if (run_linear(this, l, r, T, small, s)) return 1;
        }
        const int mw = l.mix_width();
        auto output = [&] { return small ? dense_gemv(l.o, mid, mw, T, y, w, s) : dense_gemm(l.o, l.mix_e, dense_stride(mw), T, y, w, s); };
        if (beside) {  // the block reads the mixer's own input; its router's logits came with the mixer's projections
            MoeDenseExtras ex;
            ex.logits = proj + l.router_at, ex.ld = l.in->n, ex.shared_logit = c.shared_ff ? ex.logits + c.experts : nullptr;
            if (T == 1 && moe_dense_decode_sized(l.moe, 1)) ex.W = l.o, ex.mid = mid;
            else if (output()) return 1;
            else ex.add = y;
            if (experts(l, small ? h : nullptr, small ? nullptr : h_e, ex)) return 1;
            pending = y, post = NormWeights{};
            continue;
        }
        if (output()) return 1;
        pending = y, post = l.norm1b;

        if (c.mlp == LayerConfig::NONE) continue;
        if (c.mlp == LayerConfig::DENSE) {
            const jq::GatedUnit unit{c.limit, cfg.act_alpha, cfg.act_shift};
            if (one) {
                const jq::ResidualNorm nm = update(l.norm2, xo, nullptr);
                if (dense_gemv_gated(l.gate, l.up, nullptr, 0, 1, mid, c.ff, unit, s, &nm)) return 1;
                std::swap(xc, xo);
            } else {
                if (residual_norm(update(l.norm2, xc, small ? h : nullptr), type, small ? nullptr : h_e, sw, T, nullptr, s)) return 1;
                if (small ? dense_gemv_gated(l.gate, l.up, h, w, T, mid, c.ff, unit, s)
                          : dense_gemm_gated(l.gate, l.up, h_e, sw, T, l.ff_e, dense_stride(c.ff), unit, s))
                    return 1;
            }
            if (small ? dense_gemv(l.down, mid, c.ff, T, y, w, s) : dense_gemm(l.down, l.ff_e, dense_stride(c.ff), T, y, w, s)) return 1;
        } else if (one && moe_dense_fuses_norm(l.moe, T)) {
            const jq::ResidualNorm nm = update(l.norm2, xo, h);
            MoeDenseExtras ex;
            ex.pre = &nm;
            if (experts(l, h, nullptr, ex)) return 1;
            std::swap(xc, xo);
        } else {
            // the router reads the norm in f32, the experts of a many-token step in their own type
            if (residual_norm(update(l.norm2, xc, h), type, h_e, sw, T, nullptr, s)) return 1;
            if (experts(l, h, h_e, MoeDenseExtras())) return 1;
        }
        pending = y, post = l.norm2b;
    }
    if (!n_want) return 0;
    if (one) {
        const jq::ResidualNorm nm = update(final_norm, xo, nullptr);
        if (dense_gemv(head, nullptr, 0, 1, logits, vocab, s, &nm)) return 1;
        for (int i = 1; i < n_want; i++)
            HIP_TRY(hipMemcpyAsync(logits + (size_t)i * vocab, logits, vocab * sizeof(float), hipMemcpyDeviceToDevice, s));
        return 0;
    }
    const bool few = n_want <= GEMV_MAX_ROWS;
    if (residual_norm(update(final_norm, nullptr, few ? h : nullptr), type, few ? nullptr : h_e, sw, n_want, want_ids, s)) return 1;
    return few ? dense_gemv(head, h, w, n_want, logits, vocab, s) : dense_gemm(head, h_e, sw, n_want, logits, vocab, s);
}

// ---- loading ------------------------------------------------------------------------------------------

struct StackLoader {
    LayeredModel *m;
    const jq::SafeTensors &st;

    const jq::SafeTensor *find(const std::string &name, std::initializer_list<uint64_t> shape) {
        auto it = st.tensors.find(name);
        if (it == st.tensors.end()) {
            fail("%s: missing tensor `%s`", m->arch, name.c_str());
            return nullptr;
        }
        if (it->second.shape != std::vector<uint64_t>(shape)) {
            fail("%s: tensor `%s` does not have the shape the configuration implies", m->arch, name.c_str());
            return nullptr;
        }
        return &it->second;
    }
    int host(const std::string &name, std::initializer_list<uint64_t> shape, std::vector<float> *out) {
        const jq::SafeTensor *t = find(name, shape);
        if (!t) return 1;
        out->resize(t->elems);
        if (!jq::safetensor_to_f32(*t, 0, t->elems, out->data())) return fail("%s: tensor `%s` holds no floats", m->arch, name.c_str());
        return 0;
    }
    int to_device(const std::vector<float> &v, float **out) {
        if (m->device_alloc(out, v.size())) return 1;
        HIP_TRY(hipMemcpy(*out, v.data(), v.size() * sizeof(float), hipMemcpyHostToDevice));
        return 0;
    }
    int vec(const std::string &name, std::initializer_list<uint64_t> shape, float **out) {
        std::vector<float> v;
        return host(name, shape, &v) || to_device(v, out);
    }
    int norm(const std::string &name, NormWeights *out) {
        const uint64_t w = m->cfg.width;
        return vec(name, {w}, &out->w) || (!m->cfg.rms && vec(name + ".b", {w}, &out->b));
    }
    // One matrix from the named parts' rows, one after the other, in the model's element type.
    int matrix(const std::vector<std::pair<std::string, uint64_t>> &parts, uint64_t k, jq_weight **out) {
        uint64_t n = 0;
        for (const auto &p : parts) n += p.second;
        std::vector<uint8_t> rows(n * k * m->esz());
        uint8_t *at = rows.data();
        std::vector<float> buf;
        for (const auto &p : parts) {
            const jq::SafeTensor *t = find(p.first, {p.second, k});
            if (!t) return 1;
            if (m->type == JQ_TYPE_BF16 && t->type == jq::SafeTensor::BF16) {
                memcpy(at, t->data, t->elems * 2);
            } else if (m->type == JQ_TYPE_F32) {
                if (!jq::safetensor_to_f32(*t, 0, t->elems, (float *)at)) return fail("%s: tensor `%s` holds no floats", m->arch, p.first.c_str());
            } else {
                buf.resize(t->elems);
                if (!jq::safetensor_to_f32(*t, 0, t->elems, buf.data())) return fail("%s: tensor `%s` holds no floats", m->arch, p.first.c_str());
                for (uint64_t i = 0; i < t->elems; i++) {  // round to nearest even
                    uint32_t u;
                    memcpy(&u, &buf[i], 4);
                    const uint16_t b = (u & 0x7FFFFFFFu) > 0x7F800000u ? (uint16_t)(u >> 16 | 64) : (uint16_t)((u + 0x7FFFu + (u >> 16 & 1)) >> 16);
                    memcpy(at + 2 * i, &b, 2);
                }
            }
            at += t->elems * m->esz();
        }
        if (jq_upload(m->type, rows.data(), rows.size(), n, k, 0, out)) return 1;
        m->matrices.push_back(*out);
        return 0;
    }
};

int check_stack(const StackConfig &c) {
    if (!c.vocab || !c.width) return fail("%s: zero in configuration", c.arch);
    if (c.width > (uint32_t)NORM_MAX_WIDTH) return fail("%s: width %u exceeds %d", c.arch, c.width, NORM_MAX_WIDTH);
    const int n_layers = (int)c.layers.size();
    if (c.loop_start < 0 || c.loop_start > c.loop_stop || c.loop_stop > n_layers || c.loop_times < 1)
        return fail("%s: layers %d to %d of %d run %d times", c.arch, c.loop_start, c.loop_stop, n_layers, c.loop_times);
    int v_mix = -1;
    for (size_t i = 0; i < c.layers.size(); i++) {
        const LayerConfig &l = c.layers[i];
        if (l.linear()) {
            if (l.heads <= 0 || l.dim <= 0 || l.vdim <= 0) return fail("%s: layer %zu: zero in the mixer", c.arch, i);
            if (l.dim > jq::LIN_MAX_DIM) return fail("%s: layer %zu: heads of %d exceed %d", c.arch, i, l.dim, jq::LIN_MAX_DIM);
            if (l.mixer == LayerConfig::MLSTM && !(l.gate_cap > 0.0f)) return fail("%s: layer %zu: gates capped at %g", c.arch, i, l.gate_cap);
            if (l.mixer == LayerConfig::LIGHTNING && l.decay.size() != (size_t)l.heads)
                return fail("%s: layer %zu: %zu decays for %d heads", c.arch, i, l.decay.size(), l.heads);
            for (double d : l.decay)
                if (!(d >= 0.0 && d <= 1.0)) return fail("%s: layer %zu: a decay of %g", c.arch, i, d);
        } else if (l.mixer == LayerConfig::LATENT) {
            if (l.heads <= 0 || l.dim <= 0 || l.vdim <= 0 || l.q_rank <= 0 || l.kv_rank <= 0 || l.rot_dim < 0)
                return fail("%s: layer %zu: zero in the mixer", c.arch, i);
            if (l.kv_rank > jq::LAT_MAX_R) return fail("%s: layer %zu: latents of %d exceed %d", c.arch, i, l.kv_rank, jq::LAT_MAX_R);
            if (l.q_rank > NORM_MAX_WIDTH) return fail("%s: layer %zu: query latents of %d exceed %d", c.arch, i, l.q_rank, NORM_MAX_WIDTH);
            if (l.vdim > jq::ANY_MAX_DV) return fail("%s: layer %zu: value heads of %d exceed %d", c.arch, i, l.vdim, jq::ANY_MAX_DV);
            if (l.rot.dims < 0 || l.rot.dims % 2 || l.rot.dims > l.rot_dim)
                return fail("%s: layer %zu: %d of %d dimensions rotated", c.arch, i, l.rot.dims, l.rot_dim);
        } else if (l.mixer == LayerConfig::ATTENTION) {
            if (l.heads <= 0 || l.kv_heads <= 0 || l.heads % l.kv_heads || l.dim <= 0 || l.vdim <= 0)
                return fail("%s: layer %zu: %d query heads over %d kv heads of %d and %d", c.arch, i, l.heads, l.kv_heads, l.dim, l.vdim);
            if (l.vdim > jq::ANY_MAX_DV) return fail("%s: layer %zu: value heads of %d exceed %d", c.arch, i, l.vdim, jq::ANY_MAX_DV);
            if (l.rot.dims < 0 || l.rot.dims % 2 || l.rot.dims > l.dim) return fail("%s: layer %zu: %d of %d dimensions rotated", c.arch, i, l.rot.dims, l.dim);
            if (l.v_mix) {
                if (v_mix >= 0 && c.layers[v_mix].kv_heads * c.layers[v_mix].vdim != l.kv_heads * l.vdim)
                    return fail("%s: layers %d and %zu mix values of different sizes", c.arch, v_mix, i);
                if (v_mix < 0) v_mix = (int)i;
            }
        } else {
            if (l.inner <= 0 || l.state <= 0 || l.dt_rank <= 0 || l.taps <= 0) return fail("%s: layer %zu: zero in the mixer", c.arch, i);
            if (l.state > jq::SCAN_MAX_STATES) return fail("%s: layer %zu: %d states a channel exceed %d", c.arch, i, l.state, jq::SCAN_MAX_STATES);
        }
        if (l.mlp != LayerConfig::NONE && l.ff <= 0) return fail("%s: layer %zu: feed-forward of %d", c.arch, i, l.ff);
        if (c.parallel && l.mlp == LayerConfig::DENSE) return fail("%s: layer %zu: only experts run beside a mixer", c.arch, i);
        if (l.mlp == LayerConfig::MOE && (l.top <= 0 || l.top > l.experts)) return fail("%s: layer %zu: %d experts used of %d", c.arch, i, l.top, l.experts);
    }
    return 0;
}

// The cache or state of one run of layer i.
int make_run(LayeredModel *m, int i) {
    const Layer &l = m->layers[i];
    const LayerConfig &c = l.c;
    LayerRun r;
    r.layer = i;
    auto cache = [&](size_t elems, void **out) {  // zeroed: kernels read whole runs of a row
        uint8_t *p = nullptr;
        if (m->device_alloc(&p, elems * m->esz())) return fail("%s: cache allocation failed", m->arch);
        HIP_TRY(hipMemset(p, 0, elems * m->esz()));
        *out = p;
        return 0;
    };
    if (c.mixer == LayerConfig::ATTENTION) {
        const size_t rows = (size_t)c.kv_heads * m->n_ctx;
        if (cache(rows * l.DP(), &r.kc) || cache(rows * l.DVP(), &r.vc)) return 1;
    } else if (c.mixer == LayerConfig::LATENT) {
        if (cache((size_t)m->n_ctx * c.latent_pitch(), &r.kc)) return 1;
    } else {
        r.S_floats = c.linear() ? (size_t)c.heads * c.state_rows() * c.state_pitch() : (size_t)c.inner * c.state;
        r.tail_floats = c.linear() ? (size_t)c.heads : (size_t)(c.taps - 1) * c.inner;
        if (m->device_alloc(&r.S, r.S_floats) || m->device_alloc(&r.tail[0], r.tail_floats) || m->device_alloc(&r.tail[1], r.tail_floats)) return 1;
    }
    m->runs.push_back(r);
    return 0;
}

// The runs of a loaded stack, each with its cache or state, and the rotary tables.
int make_states(LayeredModel *m) {
    for (Layer &l : m->layers) {
        const LayerConfig &c = l.c;
        if (!c.rot.dims) continue;
        for (size_t r = 0; r < m->rots.size(); r++)
            if (m->rots[r].c == c.rot) l.rot = (int)r;
        if (l.rot < 0) {
            RotaryTable t;
            std::vector<double> freq;
            t.c = c.rot, t.mag = (float)rotary_frequencies(c.rot, &freq);
            if (m->device_alloc(&t.freq, freq.size())) return 1;
            HIP_TRY(hipMemcpy(t.freq, freq.data(), freq.size() * sizeof(double), hipMemcpyHostToDevice));
            l.rot = (int)m->rots.size();
            m->rots.push_back(t);
        }
    }
    const StackConfig &sc = m->cfg;
    for (int i = 0; i < sc.loop_start; i++)
        if (make_run(m, i)) return 1;
    for (int pass = 0; pass < sc.loop_times; pass++)
        for (int i = sc.loop_start; i < sc.loop_stop; i++)
            if (make_run(m, i)) return 1;
    for (int i = sc.loop_stop; i < (int)m->layers.size(); i++)
        if (make_run(m, i)) return 1;
    // layers with experts of the same sizes take turns with one set of scratch buffers
    m->moe_holder.resize(m->layers.size());
    for (size_t i = 0; i < m->layers.size(); i++) {
        Layer &l = m->layers[i];
        m->moe_holder[i] = (int)i;
        if (!l.moe) continue;
        l.moe_shares = (int)i;
        for (size_t j = 0; j < i && l.moe_shares == (int)i; j++) {
            const LayerConfig &o = m->layers[j].c;
            if (m->layers[j].moe && o.experts == l.c.experts && o.top == l.c.top && o.ff == l.c.ff && o.shared_ff == l.c.shared_ff) l.moe_shares = (int)j;
        }
    }
    return 0;
}

// ---- Bozosun --------------------------------------------------------------------------------------------
// Layer norms with bias on both sides of every sublayer and a constant on the residual branches; attention with
// interleaved rotary pairs, YaRN and values mixed with the first such layer's; selective-scan layers; clamped gated
// units g sigmoid(1.702 g) (u + 1), dense or as experts under a softmax over the chosen logits.

// Typed reads of a configuration object; the first failure is the one reported.
struct ConfigReader {
    const char *arch;
    bool ok = true;
    std::string where;

    void bad(const char *key, const char *what) {
        if (ok) fail("%s: config.json: %s%s%s %s", arch, where.c_str(), where.empty() ? "" : ".", key, what);
        ok = false;
    }
    const jq::Json *object(const jq::Json *j, const char *key) {
        const jq::Json *v = j ? j->find(key) : nullptr;
        if (!v || v->kind != jq::Json::OBJECT) {
            bad(key, "is not an object");
            return nullptr;
        }
        return v;
    }
    double number(const jq::Json *j, const char *key) {
        const jq::Json *v = j ? j->find(key) : nullptr;
        if (!v || v->kind != jq::Json::NUMBER) {
            bad(key, "is not a number");
            return 0.0;
        }
        return v->num;
    }
    int integer(const jq::Json *j, const char *key) {
        const double v = number(j, key);
        if (v != std::floor(v) || v < 0 || v > 2147483647.0) {
            bad(key, "is not a whole number");
            return 0;
        }
        return (int)v;
    }
    bool flag(const jq::Json *j, const char *key) {  // absent or null: false
        const jq::Json *v = j ? j->find(key) : nullptr;
        if (!v || v->kind == jq::Json::NUL) return false;
        if (v->kind != jq::Json::BOOL) bad(key, "is not a boolean");
        return v->b;
    }
    std::vector<double> numbers(const jq::Json *j, const char *key) {
        const jq::Json *v = j ? j->find(key) : nullptr;
        std::vector<double> out;
        if (!v || v->kind != jq::Json::ARRAY) {
            bad(key, "is not a list");
            return out;
        }
        for (const jq::Json &e : v->items) {
            if (e.kind != jq::Json::NUMBER) bad(key, "is not a list of numbers");
            out.push_back(e.num);
        }
        return out;
    }
    const jq::Json *optional(const jq::Json *j, const char *key) {
        const jq::Json *v = j ? j->find(key) : nullptr;
        return v && v->kind != jq::Json::NUL ? v : nullptr;
    }
};

int bozosun_config(const jq::Json &cfg, StackConfig *out) {
    ConfigReader r{"Bozosun"};
    StackConfig &s = *out;
    s.arch = "Bozosun";
    s.vocab = (uint32_t)r.integer(&cfg, "vocab"), s.width = (uint32_t)r.integer(&cfg, "width");
    s.residual_mult = (float)r.number(&cfg, "residual_mult");
    s.embedding_scale = (float)r.number(r.object(&cfg, "embedding"), "scale");
    s.norm_eps = (float)r.number(r.object(&cfg, "norm"), "eps");
    s.act_alpha = 1.702f, s.act_shift = 1.0f;
    const jq::Json *layers = cfg.find("layers");
    if (!layers || layers->kind != jq::Json::ARRAY) r.bad("layers", "is not a list");
    for (size_t i = 0; r.ok && i < layers->items.size(); i++) {
        const jq::Json *e = &layers->items[i];
        r.where = "layers[" + std::to_string(i) + "]";
        LayerConfig l;
        const jq::Json *type = e->find("type"), *mx = r.object(e, "mixer");
        if (!type || type->kind != jq::Json::STRING) {
            r.bad("type", "is not a string");
        } else if (type->str == "attention") {
            l.mixer = LayerConfig::ATTENTION;
            l.heads = r.integer(mx, "heads"), l.kv_heads = r.integer(mx, "kv_heads"), l.dim = r.integer(mx, "dim"), l.vdim = r.integer(mx, "vdim");
            l.scale = (float)r.number(mx, "scale"), l.v_mix = r.flag(mx, "v_mix");
            if (const jq::Json *rot = r.optional(mx, "rot")) {
                l.rot.dims = r.integer(rot, "dims"), l.rot.base = r.number(rot, "base");
                if (const jq::Json *sc = r.optional(rot, "scaling")) {
                    l.rot.yarn = true, l.rot.factor = r.number(sc, "factor"), l.rot.original = r.number(sc, "original");
                    l.rot.fast = r.number(sc, "fast"), l.rot.slow = r.number(sc, "slow");
                }
            }
        } else if (type->str == "mamba1") {
            l.mixer = LayerConfig::MAMBA1;
            l.inner = r.integer(mx, "inner"), l.state = r.integer(mx, "state"), l.dt_rank = r.integer(mx, "dt_rank"), l.taps = r.integer(mx, "conv");
        } else {
            r.bad("type", "names no mixer of this design");
        }
        if (const jq::Json *mlp = r.optional(e, "mlp")) {
            const jq::Json *kind = mlp->find("kind");
            if (kind && kind->kind == jq::Json::STRING && kind->str == "dense") {
                l.mlp = LayerConfig::DENSE;
                l.ff = r.integer(mlp, "ff"), l.limit = (float)r.number(mlp, "limit");
            } else if (kind && kind->kind == jq::Json::STRING && kind->str == "moe") {
                l.mlp = LayerConfig::MOE;
                const jq::Json *ex = r.object(mlp, "expert"), *ro = r.object(mlp, "router");
                l.ff = r.integer(ex, "ff"), l.limit = (float)r.number(ex, "limit");
                l.experts = r.integer(ro, "experts"), l.top = r.integer(ro, "top");
            } else {
                r.bad("mlp.kind", "names no feed-forward block of this design");
            }
        }
        s.layers.push_back(l);
    }
    return r.ok ? check_stack(s) : 1;
}

int bozosun_tensors(StackLoader &ld) {
    LayeredModel *m = ld.m;
    const StackConfig &c = m->cfg;
    const uint64_t w = c.width;
    if (ld.matrix({{"embed", c.vocab}}, w, &m->embed) || ld.matrix({{"head", c.vocab}}, w, &m->head) || ld.norm("final.norm", &m->final_norm))
        return 1;
    bool seen_v_mix = false;
    m->layers.resize(c.layers.size());
    for (size_t i = 0; i < c.layers.size(); i++) {
        Layer &l = m->layers[i];
        l.c = c.layers[i];
        const LayerConfig &lc = l.c;
        const std::string p = "l" + std::to_string(i) + ".", mx = p + "mix.", ml = p + "mlp.";
        if (ld.norm(p + "norm1", &l.norm1) || ld.norm(p + "norm1b", &l.norm1b)) return 1;
        if (lc.mixer == LayerConfig::ATTENTION) {
            const uint64_t nq = (uint64_t)lc.heads * lc.dim, nk = (uint64_t)lc.kv_heads * lc.dim, nv = (uint64_t)lc.kv_heads * lc.vdim;
            if (ld.matrix({{mx + "q", nq}, {mx + "k", nk}, {mx + "v", nv}}, w, &l.in) || ld.matrix({{mx + "o", w}}, (uint64_t)lc.heads * lc.vdim, &l.o))
                return 1;
            if (lc.v_mix) {
                l.v_first = !seen_v_mix, seen_v_mix = true;
                auto t = ld.st.tensors.find(mx + "vmix");  // a scalar, or a vector of one
                if (!l.v_first && (t == ld.st.tensors.end() || t->second.elems != 1 || !jq::safetensor_to_f32(t->second, 0, 1, &l.lambda)))
                    return fail("%s: `%svmix` is missing or no single number", m->arch, mx.c_str());
            }
        } else {
            const uint64_t C = lc.inner, N = lc.state, R = lc.dt_rank;
            std::vector<float> a_log;
            if (ld.matrix({{mx + "in", 2 * C}}, w, &l.in) || ld.matrix({{mx + "x", R + 2 * N}}, C, &l.wx) || ld.matrix({{mx + "dt", C}}, R, &l.wdt) ||
                ld.matrix({{mx + "o", w}}, C, &l.o) || ld.vec(mx + "conv", {C, (uint64_t)lc.taps}, &l.conv) || ld.vec(mx + "conv.b", {C}, &l.conv_b) ||
                ld.vec(mx + "dt.b", {C}, &l.dt_b) || ld.vec(mx + "D", {C}, &l.D) || ld.host(mx + "A_log", {C, N}, &a_log))
                return 1;
            for (float &v : a_log) v = (float)(-std::exp((double)v) * 1.4426950408889634);  // A log2(e)
            if (ld.to_device(a_log, &l.A_log2)) return 1;
        }
        if (lc.mlp == LayerConfig::NONE) continue;
        if (ld.norm(p + "norm2", &l.norm2) || ld.norm(p + "norm2b", &l.norm2b)) return 1;
        const uint64_t ff = lc.ff;
        if (lc.mlp == LayerConfig::DENSE) {
            if (ld.matrix({{ml + "gate", ff}}, w, &l.gate) || ld.matrix({{ml + "up", ff}}, w, &l.up) || ld.matrix({{ml + "down", w}}, ff, &l.down)) return 1;
            continue;
        }
        std::vector<std::pair<std::string, uint64_t>> g, u, d;
        for (int e = 0; e < lc.experts; e++) {
            const std::string ep = ml + "e" + std::to_string(e) + ".";
            g.emplace_back(ep + "gate", ff), u.emplace_back(ep + "up", ff), d.emplace_back(ep + "down", w);
        }
        std::vector<float> router, bias;
        if (ld.matrix(g, w, &l.gate) || ld.matrix(u, w, &l.up) || ld.matrix(d, ff, &l.down) ||
            ld.host(ml + "router", {(uint64_t)lc.experts, w}, &router) || ld.host(ml + "router.b", {(uint64_t)lc.experts}, &bias))
            return 1;
        jq_moe_config mc{};
        mc.n_expert = (uint32_t)lc.experts, mc.n_expert_used = (uint32_t)lc.top, mc.hidden = c.width, mc.inter = (uint32_t)ff;
        mc.gating = 2, mc.norm_topk = 1, mc.swiglu_clamp = lc.limit, mc.act_alpha = c.act_alpha, mc.act_up_shift = c.act_shift;
        if (jq_moe_create(&mc, router.data(), bias.data(), l.gate, l.up, l.down, nullptr, nullptr, nullptr, &l.moe)) return 1;
    }
    return 0;
}

// ---- Fasesun --------------------------------------------------------------------------------------------
// Mixer and experts side by side on one root-mean-square norm; matrix memories, constant-decay linear attention and
// latent attention with sinks and an output gate; sigmoid-routed experts (a correction for the choice alone) with a gated
// shared one; a run of layers may repeat with caches of its own a pass; the embedding is the output head.

int fasesun_config(const jq::Json &cfg, StackConfig *out) {
    ConfigReader r{"Fasesun"};
    StackConfig &s = *out;
    s.arch = "Fasesun";
    s.vocab = (uint32_t)r.integer(&cfg, "vocab"), s.width = (uint32_t)r.integer(&cfg, "width");
    s.norm_eps = (float)r.number(r.object(&cfg, "norm"), "eps");
    s.rms = s.parallel = true;
    if (const jq::Json *loop = r.optional(&cfg, "loop"))
        s.loop_start = r.integer(loop, "start"), s.loop_stop = r.integer(loop, "stop"), s.loop_times = r.integer(loop, "times");
    const jq::Json *layers = cfg.find("layers");
    if (!layers || layers->kind != jq::Json::ARRAY) r.bad("layers", "is not a list");
    for (size_t i = 0; r.ok && i < layers->items.size(); i++) {
        const jq::Json *e = &layers->items[i];
        r.where = "layers[" + std::to_string(i) + "]";
        LayerConfig l;
        const jq::Json *type = e->find("type"), *mx = r.object(e, "mixer");
        l.heads = r.integer(mx, "heads"), l.dim = r.integer(mx, "dim"), l.vdim = r.integer(mx, "vdim");
        if (!type || type->kind != jq::Json::STRING) {
            r.bad("type", "is not a string");
        } else if (type->str == "mlstm") {
            l.mixer = LayerConfig::MLSTM;
            l.gate_cap = (float)r.number(mx, "gate_cap");
        } else if (type->str == "lightning") {
            l.mixer = LayerConfig::LIGHTNING;
            l.decay = r.numbers(mx, "decay");
        } else if (type->str == "latent_attention") {
            l.mixer = LayerConfig::LATENT;
            l.q_rank = r.integer(mx, "q_rank"), l.kv_rank = r.integer(mx, "kv_rank"), l.rot_dim = r.integer(mx, "rot_dim");
            l.scale = (float)r.number(mx, "scale");
            if (const jq::Json *rot = r.optional(mx, "rot")) l.rot.dims = r.integer(rot, "dims"), l.rot.base = r.number(rot, "base");
        } else {
            r.bad("type", "names no mixer of this design");
        }
        if (const jq::Json *mlp = r.optional(e, "mlp")) {
            const jq::Json *kind = mlp->find("kind");
            if (kind && kind->kind == jq::Json::STRING && kind->str == "moe") {
                l.mlp = LayerConfig::MOE;
                const jq::Json *ro = r.object(mlp, "router");
                l.ff = r.integer(r.object(mlp, "expert"), "ff"), l.experts = r.integer(ro, "experts"), l.top = r.integer(ro, "top");
                if (const jq::Json *sh = r.optional(mlp, "shared")) l.shared_ff = r.integer(sh, "ff");
            } else {
                r.bad("mlp.kind", "names no feed-forward block of this design");
            }
        }
        s.layers.push_back(l);
    }
    return r.ok ? check_stack(s) : 1;
}

int fasesun_tensors(StackLoader &ld) {
    LayeredModel *m = ld.m;
    const StackConfig &c = m->cfg;
    const uint64_t w = c.width;
    if (ld.matrix({{"embed", c.vocab}}, w, &m->embed) || ld.norm("final.norm", &m->final_norm)) return 1;
    m->head = m->embed;
    m->layers.resize(c.layers.size());
    for (size_t i = 0; i < c.layers.size(); i++) {
        Layer &l = m->layers[i];
        l.c = c.layers[i];
        const LayerConfig &lc = l.c;
        const std::string p = "l" + std::to_string(i) + ".", mx = p + "mix.", ml = p + "mlp.";
        const uint64_t H = lc.heads, nv = H * lc.vdim, E = lc.experts;
        if (ld.norm(p + "norm1", &l.norm1) || ld.matrix({{mx + "o", w}}, nv, &l.o)) return 1;
        // everything that reads the layer's norm in one product: the mixer's projections, its gates, the router
        std::vector<std::pair<std::string, uint64_t>> in;
        if (lc.mixer == LayerConfig::LATENT) {
            const uint64_t Q = lc.q_rank, R = lc.kv_rank, rd = lc.rot_dim, d = lc.dim;
            in = {{mx + "dq", Q}, {mx + "dkv", R + rd}, {mx + "g", nv}};
            l.gate_at = (int)(Q + R + rd);
            if (ld.vec(mx + "dq.norm", {Q}, &l.dq_norm) || ld.vec(mx + "dkv.norm", {R}, &l.dkv_norm) || ld.vec(mx + "sink", {H}, &l.sink) ||
                ld.matrix({{mx + "uq", H * (d + rd)}}, Q, &l.uq) || ld.matrix({{mx + "uk", H * d}, {mx + "uv", nv}}, R, &l.ukv))
                return 1;
        } else {
            const uint64_t nk = H * lc.dim;
            in = {{mx + "q", nk}, {mx + "k", nk}, {mx + "v", nv}, {mx + "g", nv}};
            l.gate_at = (int)(2 * nk + nv);
            if (ld.vec(mx + "norm", {nv}, &l.mix_norm)) return 1;
            if (lc.mixer == LayerConfig::MLSTM) {
                in.insert(in.end(), {{mx + "i", H}, {mx + "f", H}});
                if (ld.vec(mx + "i.b", {H}, &l.i_b) || ld.vec(mx + "f.b", {H}, &l.f_b)) return 1;
            } else {
                std::vector<float> decay, log_decay;
                for (double v : lc.decay) decay.push_back((float)v), log_decay.push_back(v > 0.0 ? (float)std::log(v) : -1e4f);
                if (ld.to_device(decay, &l.decay) || ld.to_device(log_decay, &l.log_decay)) return 1;
            }
        }
        for (const auto &part : in) l.router_at += (int)part.second;
        if (lc.mlp == LayerConfig::MOE) {
            in.emplace_back(ml + "router", E);
            if (lc.shared_ff) in.emplace_back(ml + "shared.sg", 1);
        }
        if (ld.matrix(in, w, &l.in)) return 1;
        if (lc.mlp == LayerConfig::NONE) continue;
        const uint64_t ff = lc.ff, sf = lc.shared_ff;
        std::vector<std::pair<std::string, uint64_t>> g, u, d;
        for (uint64_t e = 0; e < E; e++) {
            const std::string ep = ml + "e" + std::to_string(e) + ".";
            g.emplace_back(ep + "gate", ff), u.emplace_back(ep + "up", ff), d.emplace_back(ep + "down", w);
        }
        std::vector<float> router, correction;
        jq_weight *sg = nullptr, *su = nullptr, *sd = nullptr;
        if (ld.matrix(g, w, &l.gate) || ld.matrix(u, w, &l.up) || ld.matrix(d, ff, &l.down) || ld.host(ml + "router", {E, w}, &router) ||
            ld.host(ml + "correction", {E}, &correction) ||
            (sf && (ld.matrix({{ml + "shared.gate", sf}}, w, &sg) || ld.matrix({{ml + "shared.up", sf}}, w, &su) ||
                    ld.matrix({{ml + "shared.down", w}}, sf, &sd))))
            return 1;
        jq_moe_config mc{};
        mc.n_expert = (uint32_t)E, mc.n_expert_used = (uint32_t)lc.top, mc.hidden = c.width, mc.inter = (uint32_t)ff, mc.gating = 1;
        if (jq_moe_create(&mc, router.data(), correction.data(), l.gate, l.up, l.down, sg, su, sd, &l.moe)) return 1;
    }
    return 0;
}

constexpr uint32_t DEFAULT_CONTEXT = 4096;  // where neither the caller nor the configuration names one

int load_layered(const char *path, const ModelLoadOptions &opt, int (*config)(const jq::Json &, StackConfig *), int (*tensors)(StackLoader &),
                 jq_model **out) {
    std::string err;
    jq::Json cfg;
    if (!jq::json_read_file(std::string(path) + "/config.json", &cfg, &err)) return fail("%s", err.c_str());
    auto m = std::make_unique<LayeredModel>();
    if (config(cfg, &m->cfg)) return 1;
    m->arch = m->cfg.arch, m->vocab = m->cfg.vocab, m->n_ctx = opt.n_ctx ? opt.n_ctx : DEFAULT_CONTEXT;
    m->type = opt.compute == JQ_COMPUTE_F32 ? JQ_TYPE_F32 : JQ_TYPE_BF16;
    auto st = jq::safetensors_open(std::string(path) + "/model.safetensors", &err);
    if (!st) return fail("%s", err.c_str());
    if (ensure_init()) return 1;
    StackLoader ld{m.get(), *st};
    if (tensors(ld) || make_states(m.get()) || m->init_outputs()) return 1;
    *out = m.release();
    return 0;
}

int load_bozosun(const char *path, const ModelLoadOptions &opt, jq_model **out) { return load_layered(path, opt, bozosun_config, bozosun_tensors, out); }
int load_fasesun(const char *path, const ModelLoadOptions &opt, jq_model **out) { return load_layered(path, opt, fasesun_config, fasesun_tensors, out); }

const RegisterModelArch g_register_bozosun({"Bozosun", true, load_bozosun});
const RegisterModelArch g_register_fasesun({"Fasesun", true, load_fasesun});

}  // namespace
