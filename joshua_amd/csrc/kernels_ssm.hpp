// A selective state-space mixer: short causal convolutions a channel, and the recurrence
//   S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n,   y_c = sum_n S[c, n] C_n + D_c x_c
// with its output gate.  States, step sizes and decays are f32; the carried state of a sequence is S [channels][N] and
// the convolution's last taps - 1 inputs [taps - 1][channels].
#pragma once
#include "kernels_dense.hpp"

namespace jq {

// out[t, c] = silu(b[c] + sum_j w[c, j] x[t - (taps - 1) + j, c]); inputs in front of the step come from tail_in,
// the step's last taps - 1 go to tail_out (another buffer: a step may be shorter than the tail).  A thread takes CONV_RUN
// tokens of a channel; places T .. T + taps - 2 of the grid are the new tail's.
constexpr int CONV_RUN = 8;

template <class O>
__global__ __launch_bounds__(256) void causal_conv_silu(const float *__restrict__ x, size_t ldx, const float *__restrict__ w,
                                                        const float *__restrict__ b, const float *__restrict__ tail_in,
                                                        float *__restrict__ tail_out, O *__restrict__ out, size_t ldo, int T, int C,
                                                        int taps) {
    const int c = (int)blockIdx.x * 256 + (int)threadIdx.x, t0 = (int)blockIdx.y * CONV_RUN;
    if (c >= C) return;
    // (the address is chosen, not the load)
    auto input = [&](int at) { return *(at >= 0 ? x + (size_t)at * ldx + c : tail_in + (size_t)(at + taps - 1) * C + c); };
    const int nt = min(CONV_RUN, T - t0);
    if (nt > 0) {
        float acc[CONV_RUN];
        const float bias = b[c];
#pragma unroll
        for (int u = 0; u < CONV_RUN; u++) acc[u] = bias;
        if (taps <= 4) {  // the inputs of the run once each
            float v[CONV_RUN + 3], wt[4];
#pragma unroll
            for (int i = 0; i < CONV_RUN + 3; i++) {  // v[i] is the input at t0 - 3 + i
                const int at = t0 - 3 + i;
                v[i] = input(max(min(at, T - 1), -(taps - 1)));  // (beyond either end: meets no weight, or no output)
            }
#pragma unroll
            for (int j = 0; j < 4; j++) wt[j] = j >= 4 - taps ? w[(size_t)c * taps + j - (4 - taps)] : 0.0f;  // wt[3]: the current token's
#pragma unroll
            for (int u = 0; u < CONV_RUN; u++)
#pragma unroll
                for (int j = 0; j < 4; j++) acc[u] = fmaf(wt[j], v[u + j], acc[u]);
        } else {
            for (int j = 0; j < taps; j++) {
                const float wj = w[(size_t)c * taps + j];
#pragma unroll
                for (int u = 0; u < CONV_RUN; u++)
                    if (u < nt) acc[u] = fmaf(wj, input(t0 + u - (taps - 1) + j), acc[u]);
            }
        }
#pragma unroll
        for (int u = 0; u < CONV_RUN; u++)
            if (u < nt) out[(size_t)(t0 + u) * ldo + c] = (O)silu(acc[u]);
    }
    for (int t = max(t0, T); t < min(t0 + CONV_RUN, T + taps - 1); t++) tail_out[(size_t)(t - T) * C + c] = input(t - (taps - 1));
}

// log(1 + e^v) = max(v, 0) + log1p(e^-|v|), and log1p(e) = 2 atanh(s), s = e / (2 + e) <= 1/3, by its series in s^2: a
// small result keeps its relative accuracy.
__device__ __forceinline__ float softplus(float v) {
    const float e = __builtin_amdgcn_exp2f(-1.44269504088896341f * fabsf(v)), s = e * __builtin_amdgcn_rcpf(2.0f + e), q = s * s;
    float p = fmaf(q, 1.0f / 15.0f, 1.0f / 13.0f);
    p = fmaf(q, p, 1.0f / 11.0f), p = fmaf(q, p, 1.0f / 9.0f), p = fmaf(q, p, 1.0f / 7.0f), p = fmaf(q, p, 0.2f), p = fmaf(q, p, 1.0f / 3.0f);
    return fmaxf(v, 0.0f) + 2.0f * fmaf(q * s, p, s);
}

// z sigmoid(z)
__device__ __forceinline__ float gate_silu(float z) { return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.44269504088896341f * z)); }

template <int LPC>
__device__ __forceinline__ float sum_lanes(float v) {
    if constexpr (LPC == 64) return wave_sum(v);
    else if constexpr (LPC == 32) return sum_row16(sum_xor16(v));
    else if constexpr (LPC == 16) return sum_row16(v);
    else if constexpr (LPC == 8) return sum_row8(v);
    else {
        v += dpp_f<0xB1>(v);
        v += dpp_f<0x4E>(v);
        return v;
    }
}

struct SsmScan {
    const float *dt_raw;      // [T][C]: step sizes before bias and softplus
    const float *dt_bias;     // [C]
    const float *bc;          // [T][ld_bc]: B (N) then C (N) of a token
    size_t ld_bc;
    const float *z;           // [T][ld_z]: output gate
    size_t ld_z;
    const float *A_log2;      // [C][N]: A log2(e)
    const float *D;           // [C]
    float *S;                 // [C][N]
    int T, C, N;
    size_t ldx, ldo;
};

// The recurrence over a step's tokens, LPC lanes a channel with NS states each (N <= LPC NS), tokens in runs of
// SCAN_RUN: a run's step sizes (softplus once a channel), inputs, B and C are put into LDS, the states advance in
// registers, and the run's outputs leave together, gated.
constexpr int SCAN_MAX_STATES = 512;

template <int LPC, int NS, class IO>
__global__ __launch_bounds__(256) void selective_scan(SsmScan a, const IO *__restrict__ x, IO *__restrict__ out) {
    constexpr int CPW = 256 / LPC, NP = LPC * NS, SCAN_RUN = NP <= 128 ? 32 : 4096 / NP;
    __shared__ float2 sd[SCAN_RUN][CPW];                                           // dt, dt x
    __shared__ float sy[SCAN_RUN][CPW];                                            // the states' part of the output
    __shared__ __attribute__((aligned(16))) float sb[SCAN_RUN][NP], scc[SCAN_RUN][NP];
    const int tid = threadIdx.x, ln = tid % LPC, ch = tid / LPC, c0 = (int)blockIdx.x * CPW, c = c0 + ch;
    float S[NS], A[NS];
#pragma unroll
    for (int j = 0; j < NS; j++) {
        const int n = ln * NS + j;
        const bool in = c < a.C && n < a.N;
        A[j] = in ? a.A_log2[(size_t)c * a.N + n] : 0.0f;
        S[j] = in ? a.S[(size_t)c * a.N + n] : 0.0f;
    }
    // a run's inputs travel in registers while the run before is worked on (rows past the end: read from the last one)
    constexpr int NI = (SCAN_RUN * CPW + 255) / 256, NB = (SCAN_RUN * NP + 255) / 256;
    float rdt[NI], rz[NI], rb[NB], rc[NB], bias[NI], skip[NI], zs[NI], dx[NI];
    IO rx[NI];
#pragma unroll
    for (int i = 0; i < NI; i++) {
        const int cc = min(c0 + (tid + 256 * i) % CPW, a.C - 1);
        bias[i] = a.dt_bias[cc], skip[i] = a.D[cc];
    }
    uint32_t odt[NI], ox[NI], oz[NI], obc[NB];  // this thread's places within a run
#pragma unroll
    for (int i = 0; i < NI; i++) {
        const uint32_t e = tid + 256 * i, t = e / CPW, cc = min(c0 + (int)(e % CPW), a.C - 1);
        odt[i] = t * (uint32_t)a.C + cc, ox[i] = t * (uint32_t)a.ldx + cc, oz[i] = t * (uint32_t)a.ld_z + cc;
    }
#pragma unroll
    for (int i = 0; i < NB; i++) {
        const uint32_t e = tid + 256 * i;
        obc[i] = e / NP * (uint32_t)a.ld_bc + min((int)(e % NP), a.N - 1);
    }
    auto fetch = [&](int t0) __attribute__((always_inline)) {
        if (t0 + (256 * NI - 1) / CPW < a.T && t0 + (256 * NB - 1) / NP < a.T) {  // a whole run lies ahead
            const float *pd = a.dt_raw + (size_t)t0 * a.C, *pz = a.z + (size_t)t0 * a.ld_z, *pb = a.bc + (size_t)t0 * a.ld_bc;
            const IO *px = x + (size_t)t0 * a.ldx;
#pragma unroll
            for (int i = 0; i < NI; i++) rdt[i] = pd[odt[i]], rx[i] = px[ox[i]], rz[i] = pz[oz[i]];
#pragma unroll
            for (int i = 0; i < NB; i++) rb[i] = pb[obc[i]], rc[i] = (pb + a.N)[obc[i]];
            return;
        }
#pragma unroll
        for (int i = 0; i < NI; i++) {
            const int e = tid + 256 * i, t = min(t0 + e / CPW, a.T - 1), cc = min(c0 + e % CPW, a.C - 1);
            rdt[i] = a.dt_raw[(size_t)t * a.C + cc], rx[i] = x[(size_t)t * a.ldx + cc], rz[i] = a.z[(size_t)t * a.ld_z + cc];
        }
#pragma unroll
        for (int i = 0; i < NB; i++) {
            const int e = tid + 256 * i, t = min(t0 + e / NP, a.T - 1), n = min(e % NP, a.N - 1);
            const float *p = a.bc + (size_t)t * a.ld_bc;
            rb[i] = p[n], rc[i] = p[a.N + n];
        }
    };
    fetch(0);
    for (int t0 = 0; t0 < a.T; t0 += SCAN_RUN) {
        const int nt = min(SCAN_RUN, a.T - t0);
#pragma unroll
        for (int i = 0; i < NI; i++) {
            const int e = tid + 256 * i, t = e / CPW, k = e % CPW;
            if (SCAN_RUN * CPW % 256 == 0 || e < SCAN_RUN * CPW) {
                const float dt = t < nt ? softplus(rdt[i] + bias[i]) : 0.0f, xv = (float)rx[i];  // (dt = 0 leaves the states alone)
                sd[t][k] = float2{dt, dt * xv};
                dx[i] = skip[i] * xv, zs[i] = rz[i];
            }
        }
#pragma unroll
        for (int i = 0; i < NB; i++) {
            const int e = tid + 256 * i, t = e / NP, n = e % NP;
            if (SCAN_RUN * NP % 256 == 0 || e < SCAN_RUN * NP) sb[t][n] = n < a.N ? rb[i] : 0.0f, scc[t][n] = n < a.N ? rc[i] : 0.0f;
        }
        __syncthreads();
        if (t0 + SCAN_RUN < a.T) fetch(t0 + SCAN_RUN);
        // four tokens at a time, the next four's operands on their way from LDS meanwhile
        float2 d[4];
        float B[4][NS], Cn[4][NS];
        auto operands = [&](int t) __attribute__((always_inline)) {
#pragma unroll
            for (int u = 0; u < 4; u++) {
                d[u] = sd[t + u][ch];
#pragma unroll
                for (int j = 0; j < NS; j++) B[u][j] = sb[t + u][ln * NS + j], Cn[u][j] = scc[t + u][ln * NS + j];
            }
        };
        operands(0);
        for (int t = 0; t < nt; t += 4) {
            float decay[4][NS], in[4][NS], cc[4][NS], y[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int u = 0; u < 4; u++)
#pragma unroll
                for (int j = 0; j < NS; j++)
                    decay[u][j] = __builtin_amdgcn_exp2f(d[u].x * A[j]), in[u][j] = d[u].y * B[u][j], cc[u][j] = Cn[u][j];
            operands(min(t + 4, SCAN_RUN - 4));
#pragma unroll
            for (int u = 0; u < 4; u++)
#pragma unroll
                for (int j = 0; j < NS; j++) {
                    S[j] = fmaf(decay[u][j], S[j], in[u][j]);
                    y[u] = fmaf(S[j], cc[u][j], y[u]);
                }
#pragma unroll
            for (int u = 0; u < 4; u++) y[u] = sum_lanes<LPC>(y[u]);
            if (ln == 0) {
#pragma unroll
                for (int u = 0; u < 4; u++) sy[t + u][ch] = y[u];
            }
        }
        __syncthreads();
#pragma unroll
        for (int i = 0; i < NI; i++) {
            const int e = tid + 256 * i, t = e / CPW, k = e % CPW;
            if (t < nt && c0 + k < a.C) out[(size_t)(t0 + t) * a.ldo + c0 + k] = (IO)((sy[t][k] + dx[i]) * gate_silu(zs[i]));
        }
        __syncthreads();
    }
#pragma unroll
    for (int j = 0; j < NS; j++) {
        const int n = ln * NS + j;
        if (c < a.C && n < a.N) a.S[(size_t)c * a.N + n] = S[j];
    }
}

// One token, with the projection of its step sizes in front: 16 lanes a channel take the channel's row of W_dt
// (dt = softplus(W_dt p + bias)) and then its N states.
template <class E>
__global__ __launch_bounds__(256) void selective_step(SsmScan a, const uint8_t *__restrict__ Wdt, size_t pitch, const float *__restrict__ p,
                                                      int rank, const float *__restrict__ x, float *__restrict__ out) {
    const int sub = threadIdx.x & 15, c = 16 * (int)blockIdx.x + ((int)threadIdx.x >> 4), cc = min(c, a.C - 1);
    const uint8_t *row = Wdt + (size_t)cc * pitch;
    float dot = 0.0f;
    for (int k = sub * E::CH; k < rank; k += 16 * E::CH) {
        float w[E::CH], v[E::CH];
        E::widen(chunk_of<E>(row, k), w);
        load_acts<E::CH>(p, k, rank, v);
#pragma unroll
        for (int i = 0; i < E::CH; i++) dot = fmaf(w[i], v[i], dot);
    }
    const float dt = softplus(sum_row16(dot) + a.dt_bias[cc]), xv = x[cc], dx = dt * xv;
    float y = 0.0f;
    for (int n = sub; n < a.N; n += 16) {
        const size_t at = (size_t)cc * a.N + n;
        const float S = fmaf(__builtin_amdgcn_exp2f(dt * a.A_log2[at]), a.S[at], dx * a.bc[n]);
        y = fmaf(S, a.bc[a.N + n], y);
        if (c < a.C) a.S[at] = S;
    }
    y = sum_row16(y);
    if (sub == 0 && c < a.C) out[c] = fmaf(a.D[c], xv, y) * gate_silu(a.z[c]);
}

}  // namespace jq
