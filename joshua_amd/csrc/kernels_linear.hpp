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
    int H, d, dv, rows, DP;      // rows: dv, or dv + 1 with the normaliser's; DP: d rounded up to 32, floats from a row of S to the next
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

// ---- many tokens in bf16: runs of LIN_CHUNK tokens ----
//
//   linear_prepare      q, k, v of every token in bf16, padded, and its log weights
//   linear_gates        per head: g, M and m of every token, the maximum in front of every chunk and what a chunk leaves of
//                       the state before it
//   linear_chunk_state  per chunk: sum_s exp(g_s - M_end) v_s k_s^T (the normaliser's row has v = 1)
//   linear_state_pass   per element of the state, chunk after chunk: the state in front of every chunk, in place
//   linear_chunk_out    per chunk: o_t = sum_{s <= t} exp(g_s - M_t) (q_t . k_s) v_s + exp(m_0 - M_t) S_0 q_t
//
// f32 numbers (weights, states) enter a product as the sum of two bf16 numbers; every sum is f32.
constexpr int LIN_CHUNK = 64, LIN_SEGMENT = 4096;  // tokens a launch set takes at most

struct LinearChunks {
    int H, DQ, VP, RS, T, nc;    // DQ: d rounded up to 32; VP: elements of a head's v; RS: rows of a chunk's state, rounded up to 16
    int OP;
    __bf16 *q, *k, *v;           // [T][H][DQ], [T][H][DQ], [T][H][VP]
    float *gi, *gf;              // [H][nc LIN_CHUNK]: log write and keep weights; then g and M
    float *m_at, *carry;         // [H][nc]: m in front of a chunk; the factor on the state across it
    float *S;                    // [H][nc][RS][DQ]
    float *o;                    // [T][H][OP]
};

__device__ __forceinline__ float exp_of(float v) { return __builtin_amdgcn_exp2f(1.44269504088896341f * v); }

static __global__ __launch_bounds__(256) void linear_prepare(LinearLayer a, LinearChunks c) {
    const int t = blockIdx.x;
    const float *p = a.proj + (size_t)t * a.ld;
    const int pairs = a.H * (c.DQ / 2);
    auto input = [&](float v) { return a.memory ? v : gate_silu(v); };
    for (int e = threadIdx.x; e < 2 * pairs; e += 256) {
        const int key = e >= pairs, i = e - key * pairs, h = i / (c.DQ / 2), d = 2 * (i % (c.DQ / 2));
        const float *src = p + (key ? a.k_at : a.q_at) + h * a.d;
        const float f = key ? 1.0f : a.q_scale;
        __bf16 *dst = (key ? c.k : c.q) + ((size_t)t * a.H + h) * c.DQ + d;
        const float x = src[min(d, a.d - 1)], y = src[min(d + 1, a.d - 1)];
        const __bf16 lo = (__bf16)(d < a.d ? input(x) * f : 0.0f), hi = (__bf16)(d + 1 < a.d ? input(y) * f : 0.0f);
        *(uint32_t *)dst = __builtin_bit_cast(uint16_t, lo) | (uint32_t)__builtin_bit_cast(uint16_t, hi) << 16;
    }
    for (int e = threadIdx.x; e < a.H * c.VP; e += 256) {
        const int h = e / c.VP, r = e % c.VP;
        c.v[(size_t)t * a.H * c.VP + e] = (__bf16)(r < a.dv ? input(p[a.v_at + h * a.dv + r]) : r < a.rows ? 1.0f : 0.0f);
    }
    for (int h = threadIdx.x; h < a.H; h += 256) {
        const size_t at = (size_t)h * c.nc * LIN_CHUNK + t;
        linear_gates_of(a, t, h, &c.gi[at], &c.gf[at]);
    }
}

// One workgroup of 16 waves a head, a wave a chunk at a time.
static __global__ __launch_bounds__(1024) void linear_gates(LinearLayer a, LinearChunks c) {
    constexpr int MAX = LIN_SEGMENT / LIN_CHUNK;
    __shared__ float F_end[MAX], g_top[MAX], m_at[MAX];
    const int h = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    float *gi = c.gi + (size_t)h * c.nc * LIN_CHUNK, *gf = c.gf + (size_t)h * c.nc * LIN_CHUNK;
    constexpr int PER = MAX / 16;
    float F[PER], top[PER];
#pragma unroll
    for (int u = 0; u < PER; u++) {
        const int n = wave + 16 * u, t = n * LIN_CHUNK + lane;
        if (n >= c.nc) continue;
        const bool live = t < c.T;
        float f = live ? gf[t] : 0.0f, i = live ? gi[t] : -INFINITY;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const float v = __shfl_up(f, off, 64);
            if (lane >= off) f += v;
        }
        float g = i - f, mx = g;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const float v = __shfl_up(mx, off, 64);
            if (lane >= off) mx = fmaxf(mx, v);
        }
        gi[t] = g, F[u] = f, top[u] = mx;
        if (lane == 63) F_end[n] = f, g_top[n] = mx;
    }
    __syncthreads();
    if (threadIdx.x == 0) {
        float m = a.memory ? a.m_in[h] : 0.0f;
        for (int n = 0; n < c.nc; n++) {
            m_at[n] = m;
            c.m_at[h * c.nc + n] = m;
            const float M = a.memory ? fmaxf(m, g_top[n]) : -F_end[n];
            c.carry[h * c.nc + n] = expf(m - M);
            m = F_end[n] + M;
        }
        if (a.memory) a.m_out[h] = m;
    }
    __syncthreads();
#pragma unroll
    for (int u = 0; u < PER; u++) {
        const int n = wave + 16 * u, t = n * LIN_CHUNK + lane;
        if (n >= c.nc) continue;
        const float M = a.memory ? fmaxf(m_at[n], top[u]) : -F[u];
        gf[t] = M;
        if (a.memory && t < c.T) a.mt[(size_t)t * a.H + h] = F[u] + M;
    }
}

// A thread's part of a transposed tile of 64 tokens x 64 columns.
struct TileUnit {
    int c, pair;
    __device__ __forceinline__ explicit TileUnit(int u) : c((u >> 3) & 7), pair((u & 7) + 8 * (u >> 6)) {}
};
constexpr int LIN_PROW = LIN_CHUNK * 2 + 16;  // bytes of a token's weights

// grid (chunks, runs of 64 state rows, heads)
static __global__ __launch_bounds__(256) void linear_chunk_state(LinearChunks c) {
    __shared__ __attribute__((aligned(16))) uint8_t vh[64 * TILE_COL], vl[64 * TILE_COL], kt[64 * TILE_COL];
    const int n = blockIdx.x, v0 = 64 * (int)blockIdx.y, h = blockIdx.z, tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), l16 = lane & 15, g = lane >> 4;
    const TileUnit u(tid);
    const int t0 = n * LIN_CHUNK + 2 * u.pair, ta = min(t0, c.T - 1), tb = min(t0 + 1, c.T - 1);
    const float *gi = c.gi + ((size_t)h * c.nc + n) * LIN_CHUNK;
    const float M = c.gf[((size_t)h * c.nc + n) * LIN_CHUNK + LIN_CHUNK - 1];
    {
        const float wa = exp_of(gi[2 * u.pair] - M), wb = exp_of(gi[2 * u.pair + 1] - M);  // (past the last token: 0)
        u32x4 ra{0, 0, 0, 0}, rb{0, 0, 0, 0};
        if (v0 + 8 * u.c < c.VP) {
            ra = *(const u32x4 *)(c.v + ((size_t)ta * c.H + h) * c.VP + v0 + 8 * u.c);
            rb = *(const u32x4 *)(c.v + ((size_t)tb * c.H + h) * c.VP + v0 + 8 * u.c);
        }
        float fa[8], fb[8];
        ElemBf16::widen(ra, fa), ElemBf16::widen(rb, fb);
#pragma unroll
        for (int e = 0; e < 8; e++) {
            const float x = wa * fa[e], y = wb * fb[e];
            const __bf16 xh = (__bf16)x, yh = (__bf16)y, xl = (__bf16)(x - (float)xh), yl = (__bf16)(y - (float)yh);
            const int at = tile_word(u.c, e, u.pair);
            *(uint32_t *)(vh + at) = __builtin_bit_cast(uint16_t, xh) | (uint32_t)__builtin_bit_cast(uint16_t, yh) << 16;
            *(uint32_t *)(vl + at) = __builtin_bit_cast(uint16_t, xl) | (uint32_t)__builtin_bit_cast(uint16_t, yl) << 16;
        }
    }
    const __bf16 *ka = c.k + ((size_t)ta * c.H + h) * c.DQ, *kb = c.k + ((size_t)tb * c.H + h) * c.DQ;
    const int vrow = v0 + 16 * wave + l16;
    float *out = c.S + (((size_t)h * c.nc + n) * c.RS + min(vrow, c.RS - 1)) * c.DQ;
    for (int d0 = 0; d0 < c.DQ; d0 += 64) {
        const bool in = d0 + 8 * u.c < c.DQ;
        const u32x4 ra = *(const u32x4 *)(ka + (in ? d0 + 8 * u.c : 0)), rb = *(const u32x4 *)(kb + (in ? d0 + 8 * u.c : 0));
        if (d0) __syncthreads();
        tile_put(kt, u.c, u.pair, ra, rb);
        __syncthreads();
        f32x4 acc[4];
#pragma unroll
        for (int i = 0; i < 4; i++) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < 2; ks++) {
            const int vat = tile_chunk(16 * wave + l16, 4 * ks + g);
            const u32x4 fh = *(const u32x4 *)(vh + vat), fl = *(const u32x4 *)(vl + vat);
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const u32x4 fk = *(const u32x4 *)(kt + tile_chunk(16 * i + l16, 4 * ks + g));
                acc[i] = ElemBf16::mma(fk, fh, acc[i]);
                acc[i] = ElemBf16::mma(fk, fl, acc[i]);
            }
        }
        if (vrow < c.RS) {
#pragma unroll
            for (int i = 0; i < 4; i++)
                if (d0 + 16 * i < c.DQ) *(f32x4 *)(out + d0 + 16 * i + 4 * g) = acc[i];
        }
    }
}

// A thread has four elements of a head's state: S is the sequence's, [H][rows][DP].
static __global__ __launch_bounds__(256) void linear_state_pass(LinearChunks c, float *__restrict__ S, int rows) {
    const int per = rows * (c.DQ / 4), e = (int)blockIdx.x * 256 + (int)threadIdx.x, h = blockIdx.y;
    if (e >= per) return;
    f32x4 *state = (f32x4 *)(S + (size_t)h * rows * c.DQ) + e;
    const size_t step = (size_t)c.RS * c.DQ / 4;
    f32x4 *p = (f32x4 *)(c.S + (size_t)h * c.nc * c.RS * c.DQ) + e;
    const float *carry = c.carry + h * c.nc;
    f32x4 s = *state, next[4];
#pragma unroll
    for (int i = 0; i < 4; i++) next[i] = p[min(i, c.nc - 1) * step];
    for (int n = 0; n < c.nc; n += 4) {
        f32x4 now[4];
#pragma unroll
        for (int i = 0; i < 4; i++) now[i] = next[i];
#pragma unroll
        for (int i = 0; i < 4; i++) next[i] = p[min(n + 4 + i, c.nc - 1) * step];  // (the last one again past the end)
#pragma unroll
        for (int i = 0; i < 4; i++) {
            if (n + i < c.nc) {
                p[(n + i) * step] = s;
                const float f = carry[n + i];
#pragma unroll
                for (int r = 0; r < 4; r++) s[r] = fmaf(f, s[r], now[i][r]);
            }
        }
    }
    *state = s;
}

// x as the sum of two bf16 numbers, for eight elements.
__device__ __forceinline__ void split_bf16(const f32x4 &a, const f32x4 &b, u32x4 *hi, u32x4 *lo) {
    const bf16x4 ha = __builtin_convertvector(a, bf16x4), hb = __builtin_convertvector(b, bf16x4);
    const bf16x4 la = __builtin_convertvector(a - __builtin_convertvector(ha, f32x4), bf16x4);
    const bf16x4 lb = __builtin_convertvector(b - __builtin_convertvector(hb, f32x4), bf16x4);
    const uint2 h0 = __builtin_bit_cast(uint2, ha), h1 = __builtin_bit_cast(uint2, hb), l0 = __builtin_bit_cast(uint2, la), l1 = __builtin_bit_cast(uint2, lb);
    *hi = u32x4{h0.x, h0.y, h1.x, h1.y}, *lo = u32x4{l0.x, l0.y, l1.x, l1.y};
}

// grid (chunks, runs of 64 VT state rows, heads).  q and k pass through LDS in blocks of 64 columns.  Wave w has the weights
// of tokens 16 w .. 16 w + 15, and 16 VT of the run's state rows for all tokens: a state is read and split once a workgroup.
template <int VT>
__global__ __launch_bounds__(256) void linear_chunk_out(LinearChunks c) {
    __shared__ __attribute__((aligned(16))) uint8_t vt[64 * VT * TILE_COL], mem[2 * 64 * LIN_PROW];
    __shared__ float gs[LIN_CHUNK], Ms[LIN_CHUNK];
    uint8_t *qs = mem, *ks = mem + 64 * 128, *ph = mem, *pl = mem + 64 * LIN_PROW;  // (the weights come when q and k are through)
    const int n = blockIdx.x, v0 = 64 * VT * (int)blockIdx.y, h = blockIdx.z, tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), l16 = lane & 15, g = lane >> 4;
    const size_t at = ((size_t)h * c.nc + n) * LIN_CHUNK;
    if (tid < LIN_CHUNK) gs[tid] = c.gi[at + tid], Ms[tid] = c.gf[at + tid];
    // row r of a block: eight chunks of 16 bytes, chunk j at place j ^ (r & 7)
    const int r0 = tid >> 3, ch = tid & 7;
    const size_t row0 = ((size_t)min(n * LIN_CHUNK + r0, c.T - 1) * c.H + h) * c.DQ, row1 = ((size_t)min(n * LIN_CHUNK + r0 + 32, c.T - 1) * c.H + h) * c.DQ;
    const int place = 16 * (ch ^ (r0 & 7));
    u32x4 pre[4];
    auto fetch = [&](int d) __attribute__((always_inline)) {
        const int col = d + 8 * ch < c.DQ ? d + 8 * ch : 0;
        pre[0] = *(const u32x4 *)(c.q + row0 + col), pre[1] = *(const u32x4 *)(c.q + row1 + col);
        pre[2] = *(const u32x4 *)(c.k + row0 + col), pre[3] = *(const u32x4 *)(c.k + row1 + col);
    };
    fetch(0);
    const float *sr[VT];
#pragma unroll
    for (int j = 0; j < VT; j++) sr[j] = c.S + (((size_t)h * c.nc + n) * c.RS + min(v0 + 16 * (VT * wave + j) + l16, c.RS - 1)) * c.DQ + 8 * g;
    f32x4 state[VT][4];  // 64 columns of this wave's rows
    auto fetch_state = [&](int d) __attribute__((always_inline)) {
#pragma unroll
        for (int j = 0; j < VT; j++) {
            state[j][0] = *(const f32x4 *)(sr[j] + d), state[j][1] = *(const f32x4 *)(sr[j] + d + 4);
            if (d + 32 < c.DQ) state[j][2] = *(const f32x4 *)(sr[j] + d + 32), state[j][3] = *(const f32x4 *)(sr[j] + d + 36);
        }
    };
    fetch_state(0);
    {
        const TileUnit u(tid);
        const int t0 = n * LIN_CHUNK + 2 * u.pair, ta = min(t0, c.T - 1), tb = min(t0 + 1, c.T - 1);
#pragma unroll
        for (int j = 0; j < VT; j++) {
            const int col = v0 + 64 * j + 8 * u.c;
            u32x4 ra{0, 0, 0, 0}, rb{0, 0, 0, 0};
            if (col < c.VP) {
                ra = *(const u32x4 *)(c.v + ((size_t)ta * c.H + h) * c.VP + col);
                rb = *(const u32x4 *)(c.v + ((size_t)tb * c.H + h) * c.VP + col);
            }
            tile_put(vt + 64 * j * TILE_COL, u.c, u.pair, ra, rb);
        }
    }
    f32x4 st[4], from[VT][4];
#pragma unroll
    for (int i = 0; i < 4; i++) {
        st[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < VT; j++) from[j][i] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    for (int d = 0; d < c.DQ; d += 64) {
        if (d) __syncthreads();
        *(u32x4 *)(qs + r0 * 128 + place) = pre[0], *(u32x4 *)(qs + (r0 + 32) * 128 + place) = pre[1];
        *(u32x4 *)(ks + r0 * 128 + place) = pre[2], *(u32x4 *)(ks + (r0 + 32) * 128 + place) = pre[3];
        __syncthreads();
        u32x4 hi[VT][2], lo[VT][2];
#pragma unroll
        for (int j = 0; j < VT; j++)
#pragma unroll
            for (int kk = 0; kk < 2; kk++) split_bf16(state[j][2 * kk], state[j][2 * kk + 1], &hi[j][kk], &lo[j][kk]);
        if (d + 64 < c.DQ) fetch(d + 64), fetch_state(d + 64);
#pragma unroll
        for (int kk = 0; kk < 2; kk++) {
            if (d + 32 * kk >= c.DQ) break;
            const int piece = 16 * ((4 * kk + g) ^ (l16 & 7));
            u32x4 q[4];
#pragma unroll
            for (int i = 0; i < 4; i++) q[i] = *(const u32x4 *)(qs + (16 * i + l16) * 128 + piece);
            const u32x4 own = *(const u32x4 *)(qs + (16 * wave + l16) * 128 + piece);
#pragma unroll
            for (int i = 0; i < 4; i++)
                if (i <= wave) st[i] = ElemBf16::mma(*(const u32x4 *)(ks + (16 * i + l16) * 128 + piece), own, st[i]);
#pragma unroll
            for (int j = 0; j < VT; j++)
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    from[j][i] = ElemBf16::mma(hi[j][kk], q[i], from[j][i]);
                    from[j][i] = ElemBf16::mma(lo[j][kk], q[i], from[j][i]);
                }
        }
    }
    __syncthreads();
    {
        const int tl = 16 * wave + l16;
        const float M = Ms[tl];
#pragma unroll
        for (int i = 0; i < 4; i++) {  // keys 16 i + 4 g + r of token tl
            f32x4 p;
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int s = 16 * i + 4 * g + r;
                p[r] = s <= tl ? st[i][r] * exp_of(gs[s] - M) : 0.0f;
            }
            const bf16x4 hi = __builtin_convertvector(p, bf16x4), lo = __builtin_convertvector(p - __builtin_convertvector(hi, f32x4), bf16x4);
            *(uint2 *)(ph + tl * LIN_PROW + 32 * i + 8 * g) = __builtin_bit_cast(uint2, hi);
            *(uint2 *)(pl + tl * LIN_PROW + 32 * i + 8 * g) = __builtin_bit_cast(uint2, lo);
        }
    }
    __syncthreads();
    const float m0 = c.m_at[h * c.nc + n];
#pragma unroll
    for (int j = 0; j < VT; j++) {
        const int row = 16 * (VT * wave + j), col = v0 + row + 4 * g;
        if (v0 + row >= c.RS) break;  // (the wave agrees)
        f32x4 acc[4];
#pragma unroll
        for (int i = 0; i < 4; i++) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < 2; k++) {
            const u32x4 vf = *(const u32x4 *)(vt + 64 * (row / 64) * TILE_COL + tile_chunk(row % 64 + l16, 4 * k + g));
#pragma unroll
            for (int i = 2 * k; i < 4; i++) {  // (tokens in front of the run of keys have no weight there)
                acc[i] = ElemBf16::mma(vf, *(const u32x4 *)(ph + (16 * i + l16) * LIN_PROW + 64 * k + 16 * g), acc[i]);
                acc[i] = ElemBf16::mma(vf, *(const u32x4 *)(pl + (16 * i + l16) * LIN_PROW + 64 * k + 16 * g), acc[i]);
            }
        }
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int t = n * LIN_CHUNK + 16 * i + l16;
            if (t < c.T && col < c.OP) {
                const float in = exp_of(m0 - Ms[16 * i + l16]);
                f32x4 o;
#pragma unroll
                for (int r = 0; r < 4; r++) o[r] = fmaf(in, from[j][i][r], acc[i][r]);
                *(f32x4 *)(c.o + ((size_t)t * c.H + h) * c.OP + col) = o;
            }
        }
    }
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
    const float *g = a.gate + (size_t)t * a.ld + (size_t)h0 * a.dv, *w = a.w + (size_t)h0 * a.dv;
    // a thread's first columns stay in registers, everything of theirs asked for at once
    constexpr int KEEP = 4;
    float v[KEEP], gv[KEEP], wv[KEEP], ss = 0.0f;
#pragma unroll
    for (int i = 0; i < KEEP; i++) {
        const int c = min((int)threadIdx.x + BT * i, n - 1);
        v[i] = value(c), gv[i] = g[c], wv[i] = w[c];
    }
#pragma unroll
    for (int i = 0; i < KEEP; i++)
        if ((int)threadIdx.x + BT * i < n) ss = fmaf(v[i], v[i], ss);
    for (int c = (int)threadIdx.x + KEEP * BT; c < n; c += BT) {
        const float x = value(c);
        ss = fmaf(x, x, ss);
    }
    const float inv = 1.0f / sqrtf(sum_block<BT>(ss, red) / (float)n + a.eps);
    O *dst = out + (size_t)t * ldo + (size_t)h0 * a.dv;
#pragma unroll
    for (int i = 0; i < KEEP; i++) {
        const int c = (int)threadIdx.x + BT * i;
        if (c < n) dst[c] = (O)(v[i] * inv * wv[i] * sigmoid_of(gv[i]));
    }
    for (int c = (int)threadIdx.x + KEEP * BT; c < n; c += BT) dst[c] = (O)(value(c) * inv * w[c] * sigmoid_of(g[c]));
}

}  // namespace jq
