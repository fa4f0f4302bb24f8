// Linear attention with decay: per head a matrix of f32, S [rows][d], that every token multiplies by a decay and adds
// v k^T to, and that its query reads,
//   S <- keep S + write v k^T,   o = S q.
// Two mixers are of this kind:
//   constant decay  keep is a number per head, write = 1; q, k and v go through silu;
//   matrix memory   log-gates i = cap tanh((z_i + b_i) / cap), f = log sigmoid(cap tanh((z_f + b_f) / cap)) and a running
//                   maximum m (0 in front of the first token): m' = max(f + m, i), keep = exp(f + m - m'),
//                   write = exp(i - m').  S has one row more than v has elements, with v = 1 there: the normaliser n.
//                   The head's output is S q / (max(|n . q|, exp(-m)) + 1e-6).
// Over a run of tokens, with F_t the sum of f up to t and g_s = i_s - F_s, the maximum is m_t = F_t + M_t,
// M_t = max(m_0, max_{s <= t} g_s), token s weighs exp(g_s - M_t) in the output of t and the state in front of the run
// exp(m_0 - M_t): all in (0, 1], so that a run is two small matrix products.  The constant decay is the same with
// i = 0, f = log decay and M_t = -F_t (m_t = 0).
#pragma once
#include "kernels_ssm.hpp"

namespace jq {

struct LinearLayer {
    int H, d, dv, rows, DP;      // rows: dv, or dv + 1 with the normaliser's; DP: d rounded up to 4, floats from a row of S to the next
    int memory;                  // 1: gates, maximum and normaliser; 0: constant decay
    int T;
    const float *proj;           // [T][ld]: the projections of a token, in places q, k, v, zi, zf
    size_t ld;
    int q_at, k_at, v_at, i_at, f_at;
    float q_scale, cap;
    const float *i_b, *f_b;      // [H]
    const float *decay, *log_decay;  // [H]
    float *S;                    // [H][rows][DP], zeros behind the d-th
    const float *m_in;           // [H]
    float *m_out;                // [H], another buffer: a launch's workgroups all read m_in
    float *o;                    // [T][H][OP]: S q
    int OP;                      // rows rounded up to 4
    float *mt;                   // [T][H]: m
};

__device__ __forceinline__ float linear_input(const LinearLayer &a, float v) { return a.memory ? v : silu(v); }

// log write and log keep weights of token t (before the maximum).
__device__ __forceinline__ void linear_gates_of(const LinearLayer &a, int t, int h, float *i, float *f) {
    if (!a.memory) {
        *i = 0.0f, *f = a.log_decay[h];
        return;
    }
    const float *p = a.proj + (size_t)t * a.ld;
    *i = a.cap * tanhf((p[a.i_at + h] + a.i_b[h]) / a.cap);
    const float z = a.cap * tanhf((p[a.f_at + h] + a.f_b[h]) / a.cap);
    *f = fminf(z, 0.0f) - log1pf(expf(-fabsf(z)));
}

// Token after token: any step in 32-bit, short ones in any type.  A workgroup takes 256 / LPR rows of a head's S, LPR
// lanes a row with NS runs of four elements each (d <= 4 LPR NS), tokens in runs of LIN_RUN.
constexpr int LIN_MAX_DIM = 1024;

template <int LPR, int NS>
__global__ __launch_bounds__(256) void linear_steps(LinearLayer a) {
    constexpr int RPW = 256 / LPR, DC = 4 * LPR * NS, LIN_RUN = DC > 512 ? 4 : 8;
    __shared__ __attribute__((aligned(16))) float sq[LIN_RUN][DC], sk[LIN_RUN][DC];
    __shared__ float sv[LIN_RUN][RPW], si[LIN_RUN], sf[LIN_RUN];
    const int tid = threadIdx.x, ln = tid % LPR, rr = tid / LPR, h = blockIdx.y, row = (int)blockIdx.x * RPW + rr;
    const bool live = row < a.rows;
    float *Sr = a.S + ((size_t)h * a.rows + min(row, a.rows - 1)) * a.DP;
    float S[NS][4];
#pragma unroll
    for (int j = 0; j < NS; j++) {
        const int c = 4 * (ln + LPR * j);
        const float4 v = c < a.DP ? *(const float4 *)(Sr + c) : float4{0.f, 0.f, 0.f, 0.f};
        S[j][0] = v.x, S[j][1] = v.y, S[j][2] = v.z, S[j][3] = v.w;
    }
    float m = a.memory ? a.m_in[h] : 0.0f;
    const float decay = a.memory ? 0.0f : a.decay[h];
    for (int t0 = 0; t0 < a.T; t0 += LIN_RUN) {
        const int nt = min(LIN_RUN, a.T - t0);
        if (t0) __syncthreads();
        for (int e = tid; e < nt * DC; e += 256) {
            const int t = e / DC, c = e % DC;
            const float *p = a.proj + (size_t)(t0 + t) * a.ld;
            sq[t][c] = c < a.d ? linear_input(a, p[a.q_at + h * a.d + c]) * a.q_scale : 0.0f;
            sk[t][c] = c < a.d ? linear_input(a, p[a.k_at + h * a.d + c]) : 0.0f;
        }
        for (int e = tid; e < nt * RPW; e += 256) {
            const int t = e / RPW, r = (int)blockIdx.x * RPW + e % RPW;
            sv[t][e % RPW] = r < a.dv ? linear_input(a, a.proj[(size_t)(t0 + t) * a.ld + a.v_at + h * a.dv + r]) : 1.0f;
        }
        if (a.memory && tid < nt) linear_gates_of(a, t0 + tid, h, &si[tid], &sf[tid]);
        __syncthreads();
        for (int t = 0; t < nt; t++) {
            float keep, write = 1.0f;
            if (a.memory) {
                const float m_new = fmaxf(sf[t] + m, si[t]);
                keep = expf(sf[t] + m - m_new), write = expf(si[t] - m_new), m = m_new;
                if (blockIdx.x == 0 && tid == 0) a.mt[(size_t)(t0 + t) * a.H + h] = m;
            } else {
                keep = decay;
            }
            const float v = write * sv[t][rr];
            float o = 0.0f;
#pragma unroll
            for (int j = 0; j < NS; j++) {
                const int c = 4 * (ln + LPR * j);
                const float4 k = *(const float4 *)&sk[t][c], q = *(const float4 *)&sq[t][c];
                S[j][0] = fmaf(keep, S[j][0], v * k.x), o = fmaf(S[j][0], q.x, o);
                S[j][1] = fmaf(keep, S[j][1], v * k.y), o = fmaf(S[j][1], q.y, o);
                S[j][2] = fmaf(keep, S[j][2], v * k.z), o = fmaf(S[j][2], q.z, o);
                S[j][3] = fmaf(keep, S[j][3], v * k.w), o = fmaf(S[j][3], q.w, o);
            }
            o = sum_lanes<LPR>(o);
            if (ln == 0 && live) a.o[((size_t)(t0 + t) * a.H + h) * a.OP + row] = o;
        }
    }
    if (live) {
#pragma unroll
        for (int j = 0; j < NS; j++) {
            const int c = 4 * (ln + LPR * j);
            if (c < a.DP) *(float4 *)(Sr + c) = float4{S[j][0], S[j][1], S[j][2], S[j][3]};
        }
    }
    if (a.memory && blockIdx.x == 0 && tid == 0) a.m_out[h] = m;
}

// The mixer's output rows out of S q: the matrix memory's normaliser, a root mean square norm (over a head, or over all
// heads together), its weight, and the output gate.  One workgroup a (token, norm group) row.
struct LinearNorm {
    const float *o;        // [T][H][OP]
    const float *mt;       // [T][H]
    int H, dv, OP, memory, per_head;
    const float *w;        // [H dv]
    const float *gate;     // [T][ld]: before the sigmoid
    size_t ld;
    float eps;
};

template <class O, int BT>
__global__ __launch_bounds__(BT) void linear_norm_gate(LinearNorm a, O *__restrict__ out, size_t ldo) {
    __shared__ float red[BT / 64];
    const int groups = a.per_head ? a.H : 1, t = blockIdx.x / groups, h0 = a.per_head ? (int)blockIdx.x % groups : 0;
    const int n = a.per_head ? a.dv : a.H * a.dv;
    const float *src = a.o + ((size_t)t * a.H + h0) * a.OP;
    float inv_den = 1.0f;
    if (a.memory) inv_den = 1.0f / (fmaxf(fabsf(src[a.dv]), expf(-a.mt[(size_t)t * a.H + h0])) + 1e-6f);  // (per head then)
    auto value = [&](int c) { return (a.per_head ? src[c] : src[(size_t)(c / a.dv) * a.OP + c % a.dv]) * inv_den; };
    float ss = 0.0f;
    for (int c = threadIdx.x; c < n; c += BT) {
        const float v = value(c);
        ss = fmaf(v, v, ss);
    }
    const float inv = 1.0f / sqrtf(sum_block<BT>(ss, red) / (float)n + a.eps);
    const float *g = a.gate + (size_t)t * a.ld + (size_t)h0 * a.dv, *w = a.w + (size_t)h0 * a.dv;
    O *dst = out + (size_t)t * ldo + (size_t)h0 * a.dv;
    for (int c = threadIdx.x; c < n; c += BT) dst[c] = (O)(value(c) * inv * w[c] * sigmoid_of(g[c]));
}

}  // namespace jq
