// The mixture-of-experts layer object and what every kind of expert weights shares: router, gating, grouping of the
// routed pairs, combine.  How the experts' products run is a backend's business (quantized blocks: api.hip; plain
// BF16 / F32 rows: dense.hip).
#pragma once
#include "core.hpp"
#include "kernels_moe.hpp"

struct jq_moe;
namespace jqh {

// The decoder's residual add and RMSNorm in front of a layer's mixture of experts: x_out = x + res,
// hn_out = rmsnorm(x_out) w, and the experts run over hn_out.  `fused` says whether the router launch did it
// (then the caller's residual row is x_out) or a launch of its own in place (then it is still x).
struct MoePreNorm {
    jq::MoePreNormArgs a;
    bool fused;
};

struct MoeBackend {
    bool (*takes)(const jq_weight *gate, const jq_weight *up, const jq_weight *down);
    int (*reserve)(jq_moe *m, size_t T);   // scratch beside moe_reserve's
    void (*release)(jq_moe *m);            // and its end
    int (*forward)(jq_moe *m, size_t T, const float *x, float *y, hipStream_t s, MoePreNorm *pre);
};
// Backends announce themselves when the library is loaded.
struct RegisterMoeBackend {
    explicit RegisterMoeBackend(const MoeBackend *b);
};

}  // namespace jqh

struct jq_moe {
    jq_moe_config cfg;
    const jq_weight *gate, *up, *down, *sgate, *sup, *sdown;
    float *router_w = nullptr, *router_bias = nullptr;
    jq_weight *router_rows = nullptr;  // hidden not a multiple of 4 (plain-row experts): the router in padded rows
    const uint8_t **pgate = nullptr, **pup = nullptr, **pdown = nullptr;  // device tables of expert bases
    bool fold_shared = false;  // the shared expert rides along as table entry n_expert of the grouped kernels
    // scratch, grown to the largest token count seen
    size_t cap_tokens = 0;
    float *logits = nullptr, *wts = nullptr, *G = nullptr, *U = nullptr, *out = nullptr;
    float *sG = nullptr, *sU = nullptr, *sH = nullptr, *sOut = nullptr;
    uint32_t *ids = nullptr;
    int *gexp = nullptr, *offsets = nullptr, *xrow = nullptr, *yrow = nullptr;
    uint8_t *qacts = nullptr;  // activations as MFMA operand records (Q4_K experts, grouped path)
    uint8_t *gacts = nullptr;  // activations of the grouped int8 GEMM, and its tables
    int *gtab = nullptr;
    size_t gtab_rows = 0;      // row groups (and tiles) the tables hold
    int gtile_rgs = 8;         // row groups a tile of the current plan: 8 (waves share the rows), 2 (the weight rows), 0 (both: two launches)
    jq::ActsI8 qi8{nullptr, nullptr, nullptr, nullptr};  // activations as int8 planes (decode path, long rows)
    // plain-row experts: activations of the grouped GEMM, [rows][stride] in the experts' type
    uint8_t *dense_x = nullptr, *dense_act = nullptr, *dense_sact = nullptr;
    jq_weight *sgate_row = nullptr;    // the shared expert's own gate, one f32 row: its result times sigmoid(row . x)
    float *sgate_logit = nullptr;      // [tokens]
    int *group_counts = nullptr;  // grouping of long pair lists: pairs per (run, expert)
    const jqh::MoeBackend *backend = nullptr;
    std::mutex mu;
};

namespace jqh {

int moe_reserve(jq_moe *m, size_t T);
int moe_route_dev(jq_moe *m, size_t T, const float *x, hipStream_t s, jq::MoePairGroups pg,
                  jq::ActsI8 planes = jq::ActsI8{nullptr, nullptr, nullptr, nullptr}, bool *planes_made = nullptr,
                  jq::MoeGateIn *gate_later = nullptr, const jq::MoePreNormArgs *pre = nullptr);
// The gating alone: ids and weights from logits (rows gp.ld apart).
int moe_gate_dev(jq_moe *m, size_t T, const float *logits, const jq::MoeGateParams &gp, jq::MoePairGroups pg, hipStream_t s);
// The routed pairs of T tokens grouped by expert (groups 0 .. n_expert, the last one the folded shared expert's).
int moe_group_dev(jq_moe *m, size_t T, int extra, hipStream_t s);
jq::MoeGateParams moe_gate_params(const jq_moe_config &c);
// Whether the gating runs by one wave a token.
bool moe_wave_gate(const jq_moe_config &c);
void moe_swap_scratch(jq_moe *a, jq_moe *b);

}  // namespace jqh
