// Grouped-query attention over a cache in the model's element type, for any head sizes: rotary positions on interleaved
// pairs of the first dimensions of a head, value sizes of their own, and values mixed with those of an earlier layer.
// Scores, softmax weights and sums are f32 throughout; queries, keys and values are rounded to the element type once.
//
// The cache of a layer is [kv head][n_ctx][DP] keys and [kv head][n_ctx][DVP] values, head sizes rounded up to whole
// runs of 32 elements with zeros behind.
#pragma once
#include "kernels_dense.hpp"

namespace jq {

// cs[t][i] = mag (cos, sin)((pos0 + t) freq[i]), the angle formed and reduced in f64 so that far positions keep an
// f32's accuracy.
static __global__ __launch_bounds__(256) void rope_angles(const double *__restrict__ freq, int half, int pos0, int T, float mag,
                                                          float2 *__restrict__ cs) {
    const int total = T * half;
    for (int e = (int)blockIdx.x * 256 + (int)threadIdx.x; e < total; e += (int)gridDim.x * 256) {
        double s, c;
        sincos((double)(pos0 + e / half) * freq[e % half], &s, &c);
        cs[e] = float2{mag * (float)c, mag * (float)s};
    }
}

// What the kernels of one attention layer share.
struct AttnLayer {
    int H, G, d, dv;         // query heads, key / value heads, head sizes
    int DP, DVP, n_ctx;      // the cache's row sizes
    int rot;                 // dimensions rotated (pairs 2i, 2i + 1)
    float scale;
    int pos0, T;             // the step: tokens at positions pos0 .. pos0 + T - 1
    const float *qkv;        // [T][ld]: q heads, k heads, v heads of a token, as projected
    size_t ld;
    const float2 *cs;        // [T][rot / 2]
    const float *v_first;    // [T][G dv] to mix in with weight lambda, or null
    float *v_first_out;      // where this layer's own values go, or null
    float lambda;
    void *kc, *vc;
    // what the kernels for steps of many tokens know beside this
    const float *sink;       // [H]: exp(sink) joins the softmax's denominator; or null
    const float *gate;       // [T][ld_gate]: the outputs are multiplied by its sigmoid; or null
    size_t ld_gate;
    __device__ __forceinline__ float gated(float v, int t, int col) const {  // col within [0, H dv)
        return gate ? v * sigmoid_of(gate[t * ld_gate + col]) : v;
    }
};

// Elements 2i and 2i + 1 of a head as rotated.
__device__ __forceinline__ float2 rotated_pair(const float *__restrict__ head, int i, int d, int rot, const float2 *__restrict__ cs) {
    const float u = 2 * i < d ? head[2 * i] : 0.0f, v = 2 * i + 1 < d ? head[2 * i + 1] : 0.0f;
    if (2 * i >= rot) return float2{u, v};
    const float2 r = cs[i];
    return float2{u * r.x - v * r.y, v * r.x + u * r.y};
}

__device__ __forceinline__ float mixed_value(const AttnLayer &a, int t, int col, float v) {  // col within [0, G dv)
    return a.v_first ? fmaf(a.lambda, a.v_first[(size_t)t * a.G * a.dv + col], (1.0f - a.lambda) * v) : v;
}

// Steps of many tokens: q rotated into qe [T][H][DP], k and v into the cache.  One workgroup a token.
template <class E>
__global__ __launch_bounds__(256) void attn_rope_store(AttnLayer a, typename E::T *__restrict__ qe) {
    using T = typename E::T;
    const int t = blockIdx.x, half = a.DP / 2, pos = a.pos0 + t;
    const float *row = a.qkv + (size_t)t * a.ld;
    const float2 *cs = a.cs + (size_t)t * (a.rot / 2);
    for (int e = threadIdx.x; e < (a.H + a.G) * half; e += 256) {
        const int hd = e / half, i = e % half;
        const float2 v = rotated_pair(row + (size_t)hd * a.d, i, a.d, a.rot, cs);
        T *dst = hd < a.H ? qe + ((size_t)t * a.H + hd) * a.DP : (T *)a.kc + ((size_t)(hd - a.H) * a.n_ctx + pos) * a.DP;
        dst[2 * i] = (T)v.x, dst[2 * i + 1] = (T)v.y;
    }
    const float *vrow = row + (size_t)(a.H + a.G) * a.d;
    for (int e = threadIdx.x; e < a.G * a.DVP; e += 256) {
        const int hd = e / a.DVP, c = e % a.DVP;
        float v = 0.0f;
        if (c < a.dv) {
            const int col = hd * a.dv + c;
            v = vrow[col];
            if (a.v_first_out) a.v_first_out[(size_t)t * a.G * a.dv + col] = v;
            v = mixed_value(a, t, col, v);
        }
        ((T *)a.vc)[((size_t)hd * a.n_ctx + pos) * a.DVP + c] = (T)v;
    }
}

// Any element type and head size: one workgroup per (token, query head), keys in runs of ANY_CHUNK with a running
// maximum and sum.  Values: the threads of a column share the run's keys.
constexpr int ANY_CHUNK = 1024, ANY_MAX_DV = 1024;

template <class E, class O>
__global__ __launch_bounds__(256) void attention_any(AttnLayer a, const typename E::T *__restrict__ qe, O *__restrict__ out, size_t ldo) {
    using T = typename E::T;
    extern __shared__ float sm[];  // q[DP], scores[ANY_CHUNK], red[16], sums[256]
    const int t = blockIdx.x / a.H, h = blockIdx.x % a.H, kvh = h / (a.H / a.G), n_keys = a.pos0 + t + 1, tid = threadIdx.x;
    float *qs = sm, *sc = sm + a.DP, *red = sc + ANY_CHUNK, *sums = red + 16;
    for (int c = tid; c < a.DP; c += 256) qs[c] = (float)qe[((size_t)t * a.H + h) * a.DP + c];
    __syncthreads();
    const uint8_t *kb = (const uint8_t *)((const T *)a.kc + (size_t)kvh * a.n_ctx * a.DP);
    const T *vb = (const T *)a.vc + (size_t)kvh * a.n_ctx * a.DVP;
    const int cols = min(a.dv, 256), parts = 256 / cols, part = tid / cols, col = tid % cols;
    float m_run = -INFINITY, l_run = 0.0f, acc[ANY_MAX_DV / 256] = {0.f, 0.f, 0.f, 0.f};
    for (int j0 = 0; j0 < n_keys; j0 += ANY_CHUNK) {
        const int nj = min(ANY_CHUNK, n_keys - j0);
        float mx = -INFINITY;
        for (int j = tid; j < nj; j += 256) {
            const uint8_t *kr = kb + (size_t)(j0 + j) * a.DP * sizeof(T);
            float s = 0.0f;
            for (int c = 0; c < a.DP; c += E::CH) {
                float kv[E::CH];
                E::widen(chunk_of<E>(kr, c), kv);
#pragma unroll
                for (int i = 0; i < E::CH; i++) s = fmaf(qs[c + i], kv[i], s);
            }
            s *= a.scale;
            sc[j] = s;
            mx = fmaxf(mx, s);
        }
        mx = wave_max(mx);
        __syncthreads();
        if ((tid & 63) == 0) red[tid >> 6] = mx;
        __syncthreads();
        mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
        const float m_new = fmaxf(m_run, mx), rescale = expf(m_run - m_new);
        float sum = 0.0f;
        for (int j = tid; j < nj; j += 256) {
            const float e = expf(sc[j] - m_new);
            sc[j] = e;
            sum += e;
        }
        l_run = fmaf(l_run, rescale, block_sum(sum, red));
        m_run = m_new;
        __syncthreads();
#pragma unroll
        for (int i = 0; i < ANY_MAX_DV / 256; i++) {
            const int c = col + 256 * i;
            if (part >= parts || c >= a.dv) break;
            float v = acc[i] * rescale;
            for (int j = part; j < nj; j += parts) v = fmaf(sc[j], (float)vb[(size_t)(j0 + j) * a.DVP + c], v);
            acc[i] = v;
        }
        __syncthreads();
    }
    if (a.sink) l_run += expf(a.sink[h] - m_run);
    O *op = out + (size_t)t * ldo + (size_t)h * a.dv;
#pragma unroll
    for (int i = 0; i < ANY_MAX_DV / 256; i++) {
        sums[tid] = part < parts ? acc[i] : 0.0f;
        __syncthreads();
        if (tid < cols && tid + 256 * i < a.dv) {
            float v = 0.0f;
            for (int p = 0; p < parts; p++) v += sums[p * cols + tid];
            op[tid + 256 * i] = (O)a.gated(v / l_run, t, h * a.dv + tid + 256 * i);
        }
        __syncthreads();
    }
}

// Steps of up to 8 tokens, head sizes up to DC (64, 128 or 256): one workgroup per (chunk of ATT_CHUNK keys, KV head, run of
// `per` <= DEC_HEADS of its query heads, token): several heads a workgroup where there are workgroups enough.  The chunk's keys and values are read once for those heads; the step's own
// tokens come from the raw projections, rotated and mixed here, and the workgroups of a token's last chunk store them
// into the cache.  Partial results (maximum, sum, unnormalised output) go to attention_merge.
constexpr int DEC_HEADS = 8, DEC_TOKENS = 8;

template <class E, int DC>
__global__ __launch_bounds__(256) void attention_decode(AttnLayer a, int n_chunks, int per, float *__restrict__ part) {
    using T = typename E::T;
    constexpr int CH = E::CH, KSTEPS = DC / (4 * CH), VIM = DC * E::BYTES / 64;
    __shared__ __attribute__((aligned(16))) float qs[DEC_HEADS][DC];
    __shared__ float sc[DEC_HEADS][ATT_CHUNK], ml[DEC_HEADS][2];
    __shared__ __attribute__((aligned(16))) T sk[DEC_TOKENS][DC], sv[DEC_TOKENS][DC];
    __shared__ __attribute__((aligned(16))) float red[2][256 * CH];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int gq = a.H / a.G, runs = (gq + per - 1) / per, t = blockIdx.y;
    // (ids 8 apart run on one XCD: the runs of a chunk's heads share its keys and values in that XCD's L2)
    const int tri = 8 * ((int)(blockIdx.x >> 3) / runs) + (int)(blockIdx.x & 7), run = (int)(blockIdx.x >> 3) % runs;
    if (tri >= n_chunks * a.G) return;
    const int chunk = tri % n_chunks, kvh = tri / n_chunks;
    const int h0 = kvh * gq + run * per, nh = min(per, gq - run * per);
    const int j0 = chunk * ATT_CHUNK, nj = min(ATT_CHUNK, a.pos0 + t + 1 - j0);
    const size_t pstride = (size_t)a.dv + 2;
    float *po = part + ((size_t)(t * a.H + h0) * n_chunks + chunk) * pstride;
    const size_t phead = (size_t)n_chunks * pstride;
    if (nj <= 0) {
        if (tid < nh) po[tid * phead] = -INFINITY, po[tid * phead + 1] = 0.0f;
        return;
    }
    // cached keys and values: every load goes out before anything is needed
    const int key = tid >> 2, sub = tid & 3, jk = j0 + min(key, nj - 1);
    const uint8_t *kr = (const uint8_t *)((const T *)a.kc + ((size_t)kvh * a.n_ctx + jk) * a.DP);
    u32x4 kraw[KSTEPS];
#pragma unroll
    for (int s = 0; s < KSTEPS; s++)
        if ((4 * s + sub) * CH < a.DP && jk < a.pos0) kraw[s] = chunk_of<E>(kr, (4 * s + sub) * CH);
    const int NG = a.DVP / CH, KP = 256 / NG, cg = tid % NG, kp = tid / NG, VI = (ATT_CHUNK + KP - 1) / KP;
    u32x4 vraw[VIM];
#pragma unroll
    for (int s = 0; s < VIM; s++) {
        const int j = kp + KP * s;
        if (s < VI && kp < KP && j < nj && j0 + j < a.pos0)
            vraw[s] = chunk_of<E>((const uint8_t *)((const T *)a.vc + ((size_t)kvh * a.n_ctx + j0 + j) * a.DVP), cg * CH);
    }
    const float *row = a.qkv + (size_t)t * a.ld;
    const int half = a.DP / 2, rh = a.rot / 2;
    for (int e = tid; e < nh * half; e += 256) {
        const int hd = e / half, i = e % half;
        const float2 v = rotated_pair(row + (size_t)(h0 + hd) * a.d, i, a.d, a.rot, a.cs + (size_t)t * rh);
        qs[hd][2 * i] = (float)(T)v.x, qs[hd][2 * i + 1] = (float)(T)v.y;  // as a step of many tokens holds it
    }
    const int new_lo = max(j0, a.pos0), n_new = j0 + nj - new_lo;  // the step's own tokens in this chunk
    if (n_new > 0) {
        for (int e = tid; e < n_new * half; e += 256) {
            const int r = e / half, i = e % half, tt = new_lo + r - a.pos0;
            const float2 v = rotated_pair(a.qkv + (size_t)tt * a.ld + (size_t)(a.H + kvh) * a.d, i, a.d, a.rot, a.cs + (size_t)tt * rh);
            const T x = (T)v.x, y = (T)v.y;
            sk[r][2 * i] = x, sk[r][2 * i + 1] = y;
            if (tt == t && run == 0) {
                T *dst = (T *)a.kc + ((size_t)kvh * a.n_ctx + new_lo + r) * a.DP;
                dst[2 * i] = x, dst[2 * i + 1] = y;
            }
        }
        for (int e = tid; e < n_new * a.DVP; e += 256) {
            const int r = e / a.DVP, c = e % a.DVP, tt = new_lo + r - a.pos0, col = kvh * a.dv + c;
            float v = 0.0f;
            if (c < a.dv) {
                const float own = a.qkv[(size_t)tt * a.ld + (size_t)(a.H + a.G) * a.d + col];
                if (a.v_first_out && tt == t && run == 0) a.v_first_out[(size_t)t * a.G * a.dv + col] = own;
                v = mixed_value(a, tt, col, own);
            }
            sv[r][c] = (T)v;
            if (tt == t && run == 0) ((T *)a.vc)[((size_t)kvh * a.n_ctx + new_lo + r) * a.DVP + c] = (T)v;
        }
    }
    __syncthreads();
    // scores: four lanes a key
    float kf[KSTEPS * CH];
#pragma unroll
    for (int s = 0; s < KSTEPS; s++) {
        float f[CH];
        const int c = (4 * s + sub) * CH;
        if (c < a.DP) {
            if (jk >= a.pos0) kraw[s] = chunk_of<E>((const uint8_t *)sk[jk - new_lo], c);
            E::widen(kraw[s], f);
        }
#pragma unroll
        for (int i = 0; i < CH; i++) kf[s * CH + i] = c < a.DP ? f[i] : 0.0f;
    }
    for (int h = 0; h < nh; h++) {
        float acc = 0.0f;
#pragma unroll
        for (int s = 0; s < KSTEPS; s++) {
            const int c = (4 * s + sub) * CH;
            if (c < a.DP) {
#pragma unroll
                for (int i = 0; i < CH; i += 4) {
                    const float4 q = *(const float4 *)&qs[h][c + i];
                    acc = fmaf(q.x, kf[s * CH + i], acc), acc = fmaf(q.y, kf[s * CH + i + 1], acc);
                    acc = fmaf(q.z, kf[s * CH + i + 2], acc), acc = fmaf(q.w, kf[s * CH + i + 3], acc);
                }
            }
        }
        acc += dpp_f<0xB1>(acc);
        acc += dpp_f<0x4E>(acc);
        if (sub == 0) sc[h][key] = key < nj ? acc * a.scale : -INFINITY;
    }
    __syncthreads();
    for (int h = wave; h < nh; h += 4) {
        const float v = sc[h][lane], mx = wave_max(v), e = expf(v - mx), l = wave_sum(e);
        sc[h][lane] = e;
        if (lane == 0) ml[h][0] = mx, ml[h][1] = l;
    }
    __syncthreads();
#pragma unroll
    for (int s = 0; s < VIM; s++) {
        const int j = kp + KP * s;
        if (s < VI && kp < KP && j < nj && j0 + j >= a.pos0) vraw[s] = chunk_of<E>((const uint8_t *)sv[j0 + j - new_lo], cg * CH);
    }
    for (int hb = 0; hb < nh; hb += 2) {
        const int two = min(2, nh - hb);
        if (kp < KP) {
            float acc[2][CH] = {};
#pragma unroll
            for (int s = 0; s < VIM; s++) {
                const int j = kp + KP * s;
                if (s < VI && j < nj) {
                    float f[CH];
                    E::widen(vraw[s], f);
                    const float e0 = sc[hb][j], e1 = two > 1 ? sc[hb + 1][j] : 0.0f;
#pragma unroll
                    for (int i = 0; i < CH; i++) acc[0][i] = fmaf(e0, f[i], acc[0][i]), acc[1][i] = fmaf(e1, f[i], acc[1][i]);
                }
            }
#pragma unroll
            for (int i = 0; i < CH; i++) red[0][kp * a.DVP + cg * CH + i] = acc[0][i], red[1][kp * a.DVP + cg * CH + i] = acc[1][i];
        }
        __syncthreads();
        for (int e = tid; e < two * a.dv; e += 256) {
            const int hh = e / a.dv, c = e % a.dv;
            float v = 0.0f;
            for (int p = 0; p < KP; p++) v += red[hh][p * a.DVP + c];
            po[(hb + hh) * phead + 2 + c] = v;
        }
        __syncthreads();
    }
    if (tid < nh) po[tid * phead] = ml[tid][0], po[tid * phead + 1] = ml[tid][1];
}

// Steps of many tokens in bf16, keys of up to DK and values of up to DV elements: a workgroup of four waves takes 64 QF rows, a row being one of
// the gq query heads of a KV head at one token (row = token gq + head), so the heads share the keys and values staged.
// Keys go by in tiles of KT.  Per tile and 16 rows:
//   S^T = K Q^T            (lane: one row's scores of the keys 4 g + r, g = lane / 16)
//   running maximum and sum per row; p = 2^(s - max)
//   O^T += V^T P^T         (values transposed on their way into LDS, the keys of a run of 32 in the order in which the
//                           lanes hold their p: place 8 g + r for key 4 g + r, 8 g + 4 + r for key 16 + 4 g + r)
// The weights p go into the second product as the sum of two bf16 numbers (16 bits of mantissa).
template <int DK, int DV, int QF, int KT>
__global__ __launch_bounds__(256, 2) void attention_tiles_bf16(AttnLayer a, const __bf16 *__restrict__ qe, __bf16 *__restrict__ out,
                                                               size_t ldo, float scale_log2) {
    constexpr int KCH = DK / 8, KROW = DK * 2, VROW = KT * 2 + 16, NK = KT * KCH / 256, NVU = KT / 2 * (DV / 8) / 256, DT = DV / 16, NF = KT / 16;
    static_assert(NK * 256 == KT * KCH && NVU * 256 == KT / 2 * (DV / 8) && DV % 64 == 0, "whole loads a thread");
    __shared__ __attribute__((aligned(16))) uint8_t ks[KT * KROW], vt[DV * VROW];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, n = lane & 15, g = lane >> 4;
    const int gq = a.H / a.G, rows = a.T * gq;
    // the rows that see the most keys first, every other run of 256 workgroups in reverse: what a compute unit gets
    // in two runs adds up evenly
    int id = (int)(blockIdx.y * gridDim.x + blockIdx.x);
    const int all = (int)(gridDim.x * gridDim.y), lo = id & ~255, hi = min(lo + 256, all);
    if (id & 256) id = lo + hi - 1 - id;
    const int kvh = id % a.G, tile = (int)gridDim.x - 1 - id / a.G;
    const int r0 = tile * 64 * QF;
    const int last_key = a.pos0 + min(r0 + 64 * QF - 1, rows - 1) / gq, first_limit = a.pos0 + r0 / gq;
    const __bf16 *kb = (const __bf16 *)a.kc + (size_t)kvh * a.n_ctx * a.DP, *vb = (const __bf16 *)a.vc + (size_t)kvh * a.n_ctx * a.DVP;

    u32x4 qf[QF][DK / 32];
    int limit[QF];
#pragma unroll
    for (int q = 0; q < QF; q++) {
        const int r = min(r0 + (wave * QF + q) * 16 + n, rows - 1), t = r / gq;
        limit[q] = a.pos0 + t;
        const uint8_t *qp = (const uint8_t *)(qe + ((size_t)t * a.H + kvh * gq + r % gq) * a.DP);
#pragma unroll
        for (int k = 0; k < DK / 32; k++) qf[q][k] = 32 * k < a.DP ? *(const u32x4 *)(qp + 64 * k + 16 * g) : u32x4{0, 0, 0, 0};
    }
    f32x4 o[QF][DT];
    float mx[QF], sum[QF];
#pragma unroll
    for (int q = 0; q < QF; q++) {
        mx[q] = -INFINITY, sum[q] = 0.0f;
#pragma unroll
        for (int d = 0; d < DT; d++) o[q][d] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    // (keys past the last one and columns past the cache's are read from within it: the former are masked, the latter
    // meet zeros of the query or are never stored)
    u32x4 kpre[NK], vpre[NVU][2];
    auto fetch = [&](int k0) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < NK; i++) {
            const int id = tid + 256 * i, row = id / KCH, c = id % KCH, key = k0 + row;
            kpre[i] = *(const u32x4 *)(kb + (size_t)min(key, last_key) * a.DP + (8 * c < a.DP ? 8 * c : 0));
        }
#pragma unroll
        for (int i = 0; i < NVU; i++) {
            const int u = tid + 256 * i, c = ((u >> 3) & 7) + 8 * ((u >> 6) % (DV / 64)), pair = (u & 7) + 8 * ((u >> 6) / (DV / 64));
#pragma unroll
            for (int b = 0; b < 2; b++) {
                const int key = k0 + 2 * pair + b;
                vpre[i][b] = *(const u32x4 *)(vb + (size_t)min(key, last_key) * a.DVP + (8 * c < a.DVP ? 8 * c : 0));
            }
        }
    };
    fetch(0);
    for (int k0 = 0; k0 <= last_key; k0 += KT) {
#pragma unroll
        for (int i = 0; i < NK; i++) {
            const int id = tid + 256 * i, row = id / KCH, c = id % KCH;
            *(u32x4 *)(ks + row * KROW + 16 * (c ^ (row & 7))) = kpre[i];
        }
#pragma unroll
        for (int i = 0; i < NVU; i++) {
            const int u = tid + 256 * i, c = ((u >> 3) & 7) + 8 * ((u >> 6) % (DV / 64)), pair = (u & 7) + 8 * ((u >> 6) / (DV / 64));
            const int run = 2 * pair / 32, k = 2 * pair % 32, at = 64 * run + 2 * (k < 16 ? 8 * (k / 4) + k % 4 : 8 * ((k - 16) / 4) + 4 + k % 4);
#pragma unroll
            for (int e = 0; e < 8; e++) {
                const uint32_t lo = vpre[i][0][e / 2], hi = vpre[i][1][e / 2];
                *(uint32_t *)(vt + (8 * c + e) * VROW + at) = e & 1 ? (lo >> 16) | (hi & 0xFFFF0000u) : (lo & 0xFFFFu) | (hi << 16);
            }
        }
        __syncthreads();
        if (k0 + KT <= last_key) fetch(k0 + KT);
        f32x4 st[QF][NF];
#pragma unroll
        for (int f = 0; f < NF; f++) {
#pragma unroll
            for (int q = 0; q < QF; q++) st[q][f] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < DK / 32; k++) {
                const u32x4 kf = *(const u32x4 *)(ks + (16 * f + n) * KROW + 16 * ((4 * k + g) ^ (n & 7)));
#pragma unroll
                for (int q = 0; q < QF; q++) st[q][f] = ElemBf16::mma(kf, qf[q][k], st[q][f]);
            }
        }
        u32x4 ph[QF][NF / 2], pl[QF][NF / 2];
#pragma unroll
        for (int q = 0; q < QF; q++) {
            float tmax = -INFINITY;
            if (k0 + KT - 1 > first_limit) {  // the tile reaches past some row's last key (all rows of a workgroup agree)
#pragma unroll
                for (int f = 0; f < NF; f++)
#pragma unroll
                    for (int r = 0; r < 4; r++)
                        if (k0 + 16 * f + 4 * g + r > limit[q]) st[q][f][r] = -INFINITY;
            }
#pragma unroll
            for (int f = 0; f < NF; f++)
#pragma unroll
                for (int r = 0; r < 4; r++) tmax = fmaxf(tmax, st[q][f][r]);
            tmax = max_xor32(max_xor16(tmax)) * scale_log2;  // (scale_log2 > 0)
            const float mnew = fmaxf(mx[q], tmax);
            // (a row that has seen no key of the tiles so far keeps its state: -inf - -inf would be NaN)
            const float base = mnew == -INFINITY ? 0.0f : mnew;
            const bool moved = mnew > mx[q];
            const float rescale = moved ? __builtin_amdgcn_exp2f(mx[q] - base) : 1.0f;
            mx[q] = mnew;
            float tsum = 0.0f;
#pragma unroll
            for (int f = 0; f < NF; f++) {
                f32x4 p;
#pragma unroll
                for (int r = 0; r < 4; r++) p[r] = __builtin_amdgcn_exp2f(fmaf(st[q][f][r], scale_log2, -base));
                tsum += (p[0] + p[1]) + (p[2] + p[3]);
                const bf16x4 hi = __builtin_convertvector(p, bf16x4), lo = __builtin_convertvector(p - __builtin_convertvector(hi, f32x4), bf16x4);
                const uint2 h2 = __builtin_bit_cast(uint2, hi), l2 = __builtin_bit_cast(uint2, lo);
                ph[q][f / 2][2 * (f & 1)] = h2.x, ph[q][f / 2][2 * (f & 1) + 1] = h2.y;
                pl[q][f / 2][2 * (f & 1)] = l2.x, pl[q][f / 2][2 * (f & 1) + 1] = l2.y;
            }
            sum[q] = fmaf(sum[q], rescale, tsum);  // this lane's keys; the four lanes of a row are added at the end
            if (__ballot(moved)) {
#pragma unroll
                for (int d = 0; d < DT; d++)
#pragma unroll
                    for (int r = 0; r < 4; r++) o[q][d][r] *= rescale;
            }
        }
#pragma unroll
        for (int d = 0; d < DT; d++) {
#pragma unroll
            for (int s = 0; s < NF / 2; s++) {
                const u32x4 vf = *(const u32x4 *)(vt + (16 * d + n) * VROW + 64 * s + 16 * g);
#pragma unroll
                for (int q = 0; q < QF; q++) {
                    o[q][d] = ElemBf16::mma(vf, ph[q][s], o[q][d]);
                    o[q][d] = ElemBf16::mma(vf, pl[q][s], o[q][d]);
                }
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int q = 0; q < QF; q++) {
        const int r = r0 + (wave * QF + q) * 16 + n;
        float total = sum_xor32(sum_xor16(sum[q]));
        if (r >= rows) continue;
        const int t = r / gq, h = kvh * gq + r % gq;
        if (a.sink) total += __builtin_amdgcn_exp2f(fmaf(a.sink[h], 1.44269504088896341f, -mx[q]));
        const float inv = 1.0f / total;
        __bf16 *op = out + (size_t)t * ldo + (size_t)h * a.dv;
#pragma unroll
        for (int d = 0; d < DT; d++)
#pragma unroll
            for (int e = 0; e < 4; e++) {
                const int c = 16 * d + 4 * g + e;
                if (c < a.dv) op[c] = (__bf16)a.gated(o[q][d][e] * inv, t, h * a.dv + c);
            }
    }
}

}  // namespace jq
