// The mixture-of-experts layer object (declared in moe.hpp; C ABI in include/joshua_hip.h).
#include "dense.hpp"

namespace jqh {

static std::vector<const MoeBackend *> &moe_backends() {
    static std::vector<const MoeBackend *> v;
    return v;
}
RegisterMoeBackend::RegisterMoeBackend(const MoeBackend *b) { moe_backends().push_back(b); }

static void moe_free_scratch(jq_moe *m) {
    for (void *p : {(void *)m->logits, (void *)m->wts, (void *)m->G, (void *)m->U, (void *)m->out, (void *)m->sG,
                    (void *)m->sU, (void *)m->sH, (void *)m->sOut, (void *)m->ids, (void *)m->gexp,
                    (void *)m->offsets, (void *)m->xrow, (void *)m->yrow, (void *)m->qacts, (void *)m->qi8.xl,
                    (void *)m->qi8.xh, (void *)m->qi8.sx, (void *)m->qi8.sxs, (void *)m->gacts, (void *)m->gtab, (void *)m->group_counts, (void *)m->sgate_logit})
        if (p) (void)hipFree(p);
    if (m->backend && m->backend->release) m->backend->release(m);
    m->qacts = nullptr;
    m->group_counts = nullptr, m->sgate_logit = nullptr;
    m->gacts = nullptr, m->gtab = nullptr, m->gtab_rows = 0;
    m->qi8 = jq::ActsI8{nullptr, nullptr, nullptr, nullptr};
    m->logits = m->wts = m->G = m->U = m->out = m->sG = m->sU = m->sH = m->sOut = nullptr;
    m->ids = nullptr;
    m->gexp = m->offsets = m->xrow = m->yrow = nullptr;
    m->cap_tokens = 0;
}

int moe_reserve(jq_moe *m, size_t T) {
    if (T <= m->cap_tokens) return 0;
    moe_free_scratch(m);
    const jq_moe_config &c = m->cfg;
    // rows of the pair buffers: the routed pairs, then one per token for a folded shared expert
    size_t P = T * c.n_expert_used, PR = P + T, groups = std::max<size_t>(PR, c.n_expert + 1) + 1;
    HIP_TRY(hipMalloc((void **)&m->logits, T * c.n_expert * sizeof(float)));
    HIP_TRY(hipMalloc((void **)&m->wts, P * sizeof(float)));
    HIP_TRY(hipMalloc((void **)&m->ids, P * sizeof(uint32_t)));
    HIP_TRY(hipMalloc((void **)&m->G, PR * c.inter * sizeof(float)));
    HIP_TRY(hipMalloc((void **)&m->U, PR * c.inter * sizeof(float)));
    HIP_TRY(hipMalloc((void **)&m->out, PR * c.hidden * sizeof(float)));
    HIP_TRY(hipMalloc((void **)&m->gexp, groups * sizeof(int)));
    HIP_TRY(hipMalloc((void **)&m->offsets, (groups + 1) * sizeof(int)));
    HIP_TRY(hipMalloc((void **)&m->xrow, PR * sizeof(int)));
    HIP_TRY(hipMalloc((void **)&m->yrow, PR * sizeof(int)));
    HIP_TRY(hipMalloc((void **)&m->group_counts, (P + jq::GROUP_RUN - 1) / jq::GROUP_RUN * c.n_expert * sizeof(int)));
    if (m->backend->reserve && m->backend->reserve(m, T)) return 1;
    if (m->sgate) {
        size_t si = m->sgate->n;
        HIP_TRY(hipMalloc((void **)&m->sG, T * si * sizeof(float)));
        HIP_TRY(hipMalloc((void **)&m->sU, T * si * sizeof(float)));
        HIP_TRY(hipMalloc((void **)&m->sH, T * si * sizeof(float)));
        HIP_TRY(hipMalloc((void **)&m->sOut, T * c.hidden * sizeof(float)));
        HIP_TRY(hipMalloc((void **)&m->sgate_logit, T * sizeof(float)));
    }
    m->cap_tokens = T;
    return 0;
}

jq::MoeGateParams moe_gate_params(const jq_moe_config &c) {
    return jq::MoeGateParams{(int)c.n_expert, (int)c.n_expert_used, (int)c.gating, (int)c.norm_topk, c.weights_scale,
                             (int)c.n_group, (int)c.topk_group, 0};
}

bool moe_wave_gate(const jq_moe_config &c) {
    static const char *no_wave = getenv("JQ_MOE_NO_WAVE_GATE");
    return !no_wave && c.n_group <= 1 && c.n_expert <= 256 && c.n_expert_used <= 64;
}

// `planes`: also leave x as fixed-point planes there (the one-expert-a-workgroup router kernel does; *planes_made
// says whether it ran)
// `gate_later`: when the gating can run by one wave a token, it is left to the caller's next kernel (the logits are
// in m->logits) and *gate_later holds its operands; else it is cleared.
// `pre`: the decoder layer's residual add and RMSNorm run inside the router launch (one token; x is then pre->hn_out,
// which that launch writes).
int moe_route_dev(jq_moe *m, size_t T, const float *x, hipStream_t s, jq::MoePairGroups pg,
                  jq::ActsI8 planes, bool *planes_made,
                  jq::MoeGateIn *gate_later, const jq::MoePreNormArgs *pre) {
    const jq_moe_config &c = m->cfg;
    const unsigned token_runs = (unsigned)((T + jq::ROUTER_TOKENS_PER_WG - 1) / jq::ROUTER_TOKENS_PER_WG);
    static const char *no_tile = getenv("JQ_MOE_NO_ROUTER_TILE");
    // (a router of a million weights or more, 256 experts of 7168: from 8 tokens, 16 us against 27)
    const size_t tile_from = (size_t)c.hidden * c.n_expert >= (1u << 20) ? 8 : 32;
    const jq::MoeGateParams gp = moe_gate_params(c);
    const bool wave_gate = moe_wave_gate(c);
    if (m->router_rows) {  // (the kernels below read a row in fours)
        const size_t E = c.n_expert, h = c.hidden, stride = dense_stride(h);
        if (pre) return fail("moe: no fused norm for rows of %u", c.hidden);
        if (T <= (size_t)GEMV_MAX_ROWS) {
            if (dense_gemv(m->router_rows, x, h, (int)T, m->logits, E, s)) return 1;
        } else {
            CallScratch scratch(1);
            uint8_t *rows = nullptr;
            if (scratch.get(T * stride * sizeof(float), s, &rows) || rows_to_elem(JQ_TYPE_F32, x, h, T, (int)h, rows, stride, s) ||
                dense_gemm(m->router_rows, rows, stride, (int)T, m->logits, E, s))
                return 1;
        }
    } else if (pre)
        hipLaunchKernelGGL(jq::moe_router_logits_norm, dim3(c.n_expert), dim3(256), 0, s, m->router_w, *pre, m->logits,
                           (int)c.hidden, (int)c.n_expert);
    else if (T >= tile_from && !no_tile)  // many tokens: a token's activations read once per eight experts (the same bits)
        hipLaunchKernelGGL(jq::moe_router_logits_tile, dim3((c.n_expert + 7) / 8, (unsigned)((T + 7) / 8)), dim3(256), 0, s,
                           m->router_w, x, m->logits, (int)T, (int)c.hidden, (int)c.n_expert,
                           c.hidden % 32 == 0 ? planes : jq::ActsI8{nullptr, nullptr, nullptr, nullptr});
    else
        hipLaunchKernelGGL(jq::moe_router_logits, dim3(c.n_expert, token_runs), dim3(256), 0, s, m->router_w, x, m->logits,
                           (int)T, (int)c.hidden, (int)c.n_expert, planes);
    if (planes_made) *planes_made = !pre && planes.xl && (c.hidden % 32 == 0 || !(T >= tile_from && !no_tile));
    if (gate_later) {
        if (wave_gate) {
            *gate_later = jq::MoeGateIn{m->logits, m->router_bias, gp, m->ids, m->wts, pg, (int)T};
            HIP_TRY(hipGetLastError());
            return 0;
        }
        gate_later->logits = nullptr;
    }
    return moe_gate_dev(m, T, m->logits, gp, pg, s);
}

int moe_gate_dev(jq_moe *m, size_t T, const float *logits, const jq::MoeGateParams &gp, jq::MoePairGroups pg, hipStream_t s) {
    const jq_moe_config &c = m->cfg;
    // no expert groups and at most 256 experts: one wave a token, reductions in registers
    if (moe_wave_gate(c)) {
        const int ne = (int)(c.n_expert + 63) / 64;
#define JQ_GATE(NE) hipLaunchKernelGGL(jq::moe_gate_topk_wave<NE>, dim3((unsigned)T), dim3(64), 0, s, logits, m->router_bias, gp, m->ids, m->wts, pg)
        if (ne == 1) JQ_GATE(1);
        else if (ne == 2) JQ_GATE(2);
        else if (ne == 3) JQ_GATE(3);
        else JQ_GATE(4);
#undef JQ_GATE
    } else {
        const size_t sm = (2 * c.n_expert + std::max<uint32_t>(c.n_group, 1) + c.n_expert_used + 4) * sizeof(float);
        hipLaunchKernelGGL(jq::moe_gate_topk, dim3((unsigned)T), dim3(256), sm, s, logits, m->router_bias, gp, m->ids, m->wts, pg);
    }
    HIP_TRY(hipGetLastError());
    return 0;
}

int moe_group_dev(jq_moe *m, size_t T, int extra, hipStream_t s) {
    const jq_moe_config &c = m->cfg;
    const int P = (int)(T * c.n_expert_used);
    const int in_lds = (size_t)P <= 12288;
    const size_t chunks = ((size_t)P + 63) / 64, rank_ints = chunks * c.n_expert + c.n_expert + 1;
    static const char *no_ranked = getenv("JQ_MOE_NO_RANKED_GROUPING");
    // (its rank table: chunks x experts ints of LDS, up to 144 KB)
    if (!no_ranked && chunks <= (size_t)jq::GROUP_RANK_CHUNKS && rank_ints <= 36864) {
        static std::once_flag big_lds;
        static hipError_t attr_rc = hipSuccess;
        std::call_once(big_lds, [&] {
            attr_rc = hipFuncSetAttribute((const void *)jq::moe_group_pairs_ranked, hipFuncAttributeMaxDynamicSharedMemorySize,
                                          36864 * (int)sizeof(int));
        });
        HIP_TRY(attr_rc);
        hipLaunchKernelGGL(jq::moe_group_pairs_ranked, dim3(1), dim3(jq::GROUP_PAIRS_THREADS), rank_ints * sizeof(int), s,
                           m->ids, (int)T, (int)c.n_expert_used, (int)c.n_expert, m->gexp, m->offsets, m->xrow, m->yrow,
                           extra);
    }
    else if (!no_ranked && (size_t)c.n_expert * (jq::GROUP_RUN / 64) * sizeof(int) <= 65536) {
        const int runs = (P + jq::GROUP_RUN - 1) / jq::GROUP_RUN, E = (int)c.n_expert;
        hipLaunchKernelGGL(jq::moe_group_count, dim3((unsigned)runs), dim3(jq::GROUP_RUN), E * sizeof(int), s, m->ids, P, E, m->group_counts);
        hipLaunchKernelGGL(jq::moe_group_starts, dim3(1), dim3(jq::GROUP_PAIRS_THREADS), (E + 1) * sizeof(int), s, m->group_counts, runs, P,
                           (int)T, E, m->gexp, m->offsets, m->xrow, m->yrow, extra);
        hipLaunchKernelGGL(jq::moe_group_place, dim3((unsigned)runs), dim3(jq::GROUP_RUN), E * (jq::GROUP_RUN / 64) * sizeof(int), s, m->ids,
                           P, (int)c.n_expert_used, E, m->group_counts, m->offsets, m->xrow, m->yrow);
    }
    else
        hipLaunchKernelGGL(jq::moe_group_pairs, dim3(1), dim3(jq::GROUP_PAIRS_THREADS), (c.n_expert + 1 + (in_lds ? P : 0)) * sizeof(int), s,
                           m->ids, (int)T, (int)c.n_expert_used, (int)c.n_expert, m->gexp, m->offsets, m->xrow, m->yrow,
                           extra, in_lds);
    return 0;
}

// Device table of expert base pointers; `extra` (the shared expert's weight, or null) becomes entry
// n_expert.
static int moe_ptr_table(const jq_weight *w, size_t n_expert, size_t rows_per_expert, const jq_weight *extra,
                  const uint8_t ***out) {
    std::vector<const uint8_t *> host(n_expert + 1);
    for (size_t e = 0; e < n_expert; e++) host[e] = w->dev + e * rows_per_expert * w->row_bytes;
    host[n_expert] = extra ? extra->dev : w->dev;
    HIP_TRY(hipMalloc((void **)out, host.size() * sizeof(uint8_t *)));
    HIP_TRY(hipMemcpy((void *)*out, host.data(), host.size() * sizeof(uint8_t *), hipMemcpyHostToDevice));
    return 0;
}

// Hands the scratch buffers of one layer object to another of the same configuration.  Work on a stream
// runs in launch order and every kernel got its pointers when it was launched, so the layers of a model
// can take turns with one set.
void moe_swap_scratch(jq_moe *a, jq_moe *b) {
    std::swap(a->cap_tokens, b->cap_tokens);
    std::swap(a->logits, b->logits), std::swap(a->wts, b->wts), std::swap(a->G, b->G), std::swap(a->U, b->U);
    std::swap(a->out, b->out), std::swap(a->sG, b->sG), std::swap(a->sU, b->sU), std::swap(a->sH, b->sH);
    std::swap(a->sOut, b->sOut), std::swap(a->ids, b->ids), std::swap(a->gexp, b->gexp);
    std::swap(a->offsets, b->offsets), std::swap(a->xrow, b->xrow), std::swap(a->yrow, b->yrow);
    std::swap(a->qacts, b->qacts), std::swap(a->gacts, b->gacts), std::swap(a->gtab, b->gtab);
    std::swap(a->dense_x, b->dense_x), std::swap(a->dense_act, b->dense_act), std::swap(a->group_counts, b->group_counts);
    std::swap(a->dense_sact, b->dense_sact), std::swap(a->sgate_logit, b->sgate_logit);
    std::swap(a->gtab_rows, b->gtab_rows), std::swap(a->gtile_rgs, b->gtile_rgs), std::swap(a->qi8, b->qi8);
}

}  // namespace jqh

extern "C" {

int jq_moe_create(const jq_moe_config *cfg, const float *router_w, const float *router_bias,
                  const jq_weight *gate_exps, const jq_weight *up_exps, const jq_weight *down_exps,
                  const jq_weight *shared_gate, const jq_weight *shared_up, const jq_weight *shared_down,
                  jq_moe **out) {
    if (!out) return fail("jq_moe_create: out is null");
    *out = nullptr;
    if (!cfg || !router_w || !gate_exps || !up_exps || !down_exps) return fail("jq_moe_create: null argument");
    const jq_moe_config &c = *cfg;
    if (c.n_expert == 0 || c.n_expert_used == 0 || c.n_expert_used > c.n_expert)
        return fail("moe: %u experts used of %u", c.n_expert_used, c.n_expert);
    if (c.gating > 2) return fail("moe: unknown gating %u", c.gating);
    if (!dense_elem_bytes(gate_exps->type) && ((c.act_alpha != 0.0f && c.act_alpha != 1.0f) || c.act_up_shift != 0.0f))
        return fail("moe: experts in block formats run SwiGLU only");
    if (c.hidden % 4 != 0 && !dense_elem_bytes(gate_exps->type)) return fail("moe: hidden size %u is not a multiple of 4", c.hidden);
    if (c.n_group > 1 && (c.n_expert % c.n_group != 0 || c.topk_group == 0 || c.topk_group > c.n_group))
        return fail("moe: %u experts in %u groups, %u groups kept", c.n_expert, c.n_group, c.topk_group);
    // reference: src/quantized_qwen3_moe.rs:567-571 (expert tensor shaped [n_expert, out, in])
    if (gate_exps->n != (size_t)c.n_expert * c.inter || gate_exps->k != c.hidden || up_exps->n != gate_exps->n ||
        up_exps->k != c.hidden || down_exps->n != (size_t)c.n_expert * c.hidden || down_exps->k != c.inter)
        return fail("moe: expected expert tensors shaped [%u*%u, %u], [%u*%u, %u], [%u*%u, %u]", c.n_expert, c.inter,
                    c.hidden, c.n_expert, c.inter, c.hidden, c.n_expert, c.hidden, c.inter);
    bool any_shared = shared_gate || shared_up || shared_down;
    if (any_shared) {
        if (!(shared_gate && shared_up && shared_down)) return fail("moe: shared expert needs gate, up and down");
        if (shared_gate->k != c.hidden || shared_up->k != c.hidden || shared_up->n != shared_gate->n ||
            shared_down->k != shared_gate->n || shared_down->n != c.hidden)
            return fail("moe: shared expert shapes do not chain");
    }
    const MoeBackend *backend = nullptr;
    for (const MoeBackend *b : moe_backends())
        if (b->takes(gate_exps, up_exps, down_exps)) backend = b;
    if (!backend) return fail("moe: no kernels for expert tensors of types %u, %u, %u", gate_exps->type, up_exps->type, down_exps->type);
    if (ensure_init()) return 1;
    jq_moe *m = new jq_moe;
    m->cfg = c;
    m->backend = backend;
    m->gate = gate_exps;
    m->up = up_exps;
    m->down = down_exps;
    m->sgate = shared_gate;
    m->sup = shared_up;
    m->sdown = shared_down;
    auto cleanup = [&] {
        jq_moe_free(m);
        return 1;
    };
    size_t rbytes = (size_t)c.n_expert * c.hidden * sizeof(float);
    if (hipMalloc((void **)&m->router_w, rbytes) != hipSuccess ||
        hipMemcpy(m->router_w, router_w, rbytes, hipMemcpyHostToDevice) != hipSuccess) {
        fail("moe: router upload failed");
        return cleanup();
    }
    if (c.hidden % 4 != 0 && jq_upload(JQ_TYPE_F32, router_w, rbytes, c.n_expert, c.hidden, 0, &m->router_rows)) return cleanup();
    if (router_bias) {
        if (hipMalloc((void **)&m->router_bias, c.n_expert * sizeof(float)) != hipSuccess ||
            hipMemcpy(m->router_bias, router_bias, c.n_expert * sizeof(float), hipMemcpyHostToDevice) != hipSuccess) {
            fail("moe: router bias upload failed");
            return cleanup();
        }
    }
    // A shared expert of the routed experts' own type and shape rides along in the grouped kernels.
    m->fold_shared = any_shared && shared_gate->type == gate_exps->type && shared_up->type == up_exps->type &&
                     shared_down->type == down_exps->type && shared_gate->n == c.inter;
    if (moe_ptr_table(gate_exps, c.n_expert, c.inter, m->fold_shared ? shared_gate : nullptr, &m->pgate) ||
        moe_ptr_table(up_exps, c.n_expert, c.inter, m->fold_shared ? shared_up : nullptr, &m->pup) ||
        moe_ptr_table(down_exps, c.n_expert, c.hidden, m->fold_shared ? shared_down : nullptr, &m->pdown))
        return cleanup();
    *out = m;
    return 0;
}

void jq_moe_free(jq_moe *m) {
    if (!m) return;
    moe_free_scratch(m);
    jq_free(m->router_rows);
    jq_free(m->sgate_row);
    for (void *p : {(void *)m->router_w, (void *)m->router_bias, (void *)m->pgate, (void *)m->pup, (void *)m->pdown})
        if (p) (void)hipFree(p);
    delete m;
}

int jq_moe_set_shared_gate(jq_moe *m, const float *row) {
    if (!m || !row) return fail("jq_moe_set_shared_gate: null argument");
    if (!m->sgate) return fail("moe: no shared expert to gate");
    if (!dense_elem_bytes(m->gate->type)) return fail("moe: a gate on the shared expert runs beside BF16 / F32 experts only");
    std::lock_guard<std::mutex> lock(m->mu);
    jq_free(m->sgate_row);
    m->sgate_row = nullptr;
    return jq_upload(JQ_TYPE_F32, row, m->cfg.hidden * sizeof(float), 1, m->cfg.hidden, 0, &m->sgate_row);
}

int jq_moe_route(jq_moe *m, size_t n_tokens, const float *x, uint32_t *ids, float *weights, int ptrs_are_device,
                 void *stream) {
    if (!m) return fail("jq_moe_route: layer is null");
    if (n_tokens == 0) return 0;
    if (!x || !ids || !weights) return fail("jq_moe_route: null pointer");
    hipStream_t s = (hipStream_t)stream;
    std::lock_guard<std::mutex> lock(m->mu);
    if (moe_reserve(m, n_tokens)) return 1;
    size_t P = n_tokens * m->cfg.n_expert_used;
    DevBuf xd;
    const float *xdev = x;
    if (!ptrs_are_device) {
        HIP_TRY(xd.alloc(n_tokens * m->cfg.hidden * sizeof(float)));
        HIP_TRY(hipMemcpyAsync(xd.p, x, n_tokens * m->cfg.hidden * sizeof(float), hipMemcpyHostToDevice, s));
        xdev = (const float *)xd.p;
    }
    if (moe_route_dev(m, n_tokens, xdev, s, jq::MoePairGroups{nullptr, nullptr, nullptr, nullptr, 0})) return 1;
    hipMemcpyKind kind = ptrs_are_device ? hipMemcpyDeviceToDevice : hipMemcpyDeviceToHost;
    HIP_TRY(hipMemcpyAsync(ids, m->ids, P * sizeof(uint32_t), kind, s));
    HIP_TRY(hipMemcpyAsync(weights, m->wts, P * sizeof(float), kind, s));
    if (!ptrs_are_device) HIP_TRY(hipStreamSynchronize(s));
    return 0;
}

int jq_moe_forward(jq_moe *m, size_t n_tokens, const float *x, float *y, int ptrs_are_device, void *stream) {
    if (!m) return fail("jq_moe_forward: layer is null");
    if (n_tokens == 0) return 0;
    if (!x || !y) return fail("jq_moe_forward: null pointer");
    hipStream_t s = (hipStream_t)stream;
    std::lock_guard<std::mutex> lock(m->mu);
    if (moe_reserve(m, n_tokens)) return 1;
    if (ptrs_are_device) return m->backend->forward(m, n_tokens, x, y, s, nullptr);
    size_t bytes = n_tokens * m->cfg.hidden * sizeof(float);
    DevBuf xd, yd;
    HIP_TRY(xd.alloc(bytes));
    HIP_TRY(yd.alloc(bytes));
    HIP_TRY(hipMemcpyAsync(xd.p, x, bytes, hipMemcpyHostToDevice, s));
    if (m->backend->forward(m, n_tokens, (const float *)xd.p, (float *)yd.p, s, nullptr)) return 1;
    HIP_TRY(hipMemcpyAsync(y, yd.p, bytes, hipMemcpyDeviceToHost, s));
    HIP_TRY(hipStreamSynchronize(s));
    return 0;
}

}  // extern "C"
