// Latent attention over a cache in the model's element type: a token leaves one row [latent | rotated shared key] for all
// heads, the latent root-mean-square normed; a head's unrotated keys are W_uk c and its values W_uv c.  Two forms:
//   short steps  the query goes into the latent's space (q W_uk), heads share the rows as keys and their first R elements as
//                values, and W_uv is applied to the weighted sum of latents;
//   long steps   keys and values of all cached tokens are written out per head, and the step runs on the kernels of
//                kernels_attention.hpp.
// Scores, softmax and sums are f32; the softmax's denominator may hold a learned sink per head.
#pragma once
#include "kernels_attention.hpp"

namespace jq {

struct LatentLayer {
    int H, d, rd, dv, R;         // heads; a query's unrotated and rotated parts; value size; latent size
    int RP, n_ctx;               // the cache's row: R + rd elements, RP apart
    int rot;                     // dimensions of the rotated part that turn
    int pos0, T;
    float scale, eps;
    const float *q;              // [T][H (d + rd)], as projected
    const float *down;           // [T][ld]: R + rd numbers a token, as projected
    size_t ld;
    const float2 *cs;            // [T][rot / 2]
    const float *norm_w;         // [R]
    const float *sink;           // [H] or null
    const float *gate;           // [T][ld]: output gate before its sigmoid, H dv numbers a token
    void *cache;                 // [n_ctx][RP]
};

// One token's row into the cache, by a workgroup of 256.
template <class E>
__device__ __forceinline__ void latent_store_row(const LatentLayer &a, int t, float *red) {
    using T = typename E::T;
    const float *x = a.down + (size_t)t * a.ld;
    T *row = (T *)a.cache + (size_t)(a.pos0 + t) * a.RP;
    float ss = 0.0f;
    for (int c = threadIdx.x; c < a.R; c += 256) ss = fmaf(x[c], x[c], ss);
    const float inv = 1.0f / sqrtf(sum_block<256>(ss, red) / (float)a.R + a.eps);
    for (int c = threadIdx.x; c < a.R; c += 256) row[c] = (T)(x[c] * inv * a.norm_w[c]);
    for (int i = threadIdx.x; i < (a.rd + 1) / 2; i += 256) {
        const float2 v = rotated_pair(x + a.R, i, a.rd, a.rot, a.cs + (size_t)t * (a.rot / 2));
        row[a.R + 2 * i] = (T)v.x;
        if (2 * i + 1 < a.rd) row[a.R + 2 * i + 1] = (T)v.y;
    }
}

template <class E>
__global__ __launch_bounds__(256) void latent_store(LatentLayer a) {
    __shared__ float red[4];
    latent_store_row<E>(a, (int)blockIdx.x, red);
}

// ---- short steps ----

// qx[t, h] = [W_uk[h]^T q | rotated q], RP numbers a row (zeros behind): grid (column runs of 16 chunks, heads + 1, tokens);
// the workgroups of the row behind the last head store the token's cache row.
template <class E>
__global__ __launch_bounds__(256) void latent_absorb(LatentLayer a, const uint8_t *__restrict__ Wuk, size_t pitch, float *__restrict__ qx) {
    constexpr int CH = E::CH;
    __shared__ float part[16][16 * CH + 1], red[4];
    const int h = blockIdx.y, t = blockIdx.z, tid = threadIdx.x;
    if (h == a.H) {
        if (blockIdx.x == 0) latent_store_row<E>(a, t, red);
        return;
    }
    const float *q = a.q + ((size_t)t * a.H + h) * (a.d + a.rd);
    float *out = qx + ((size_t)t * a.H + h) * a.RP;
    const int col = tid & 15, grp = tid >> 4, c0 = (int)blockIdx.x * 16 * CH, c = c0 + col * CH;
    float acc[CH] = {};
    if (c < a.R) {
#pragma unroll 4
        for (int r = grp; r < a.d; r += 16) {
            float w[CH];
            E::widen(chunk_of<E>(Wuk + (size_t)(h * a.d + r) * pitch, c), w);
            const float qv = q[r];
#pragma unroll
            for (int i = 0; i < CH; i++) acc[i] = fmaf(qv, w[i], acc[i]);
        }
    }
#pragma unroll
    for (int i = 0; i < CH; i++) part[grp][col * CH + i] = acc[i];
    __syncthreads();
    if (tid < 16 * CH && c0 + tid < a.R) {
        float v = 0.0f;
#pragma unroll
        for (int g = 0; g < 16; g++) v += part[g][tid];
        out[c0 + tid] = v;
    }
    if (blockIdx.x == 0) {
        for (int i = tid; i < (a.RP - a.R + 1) / 2; i += 256) {
            const float2 v = rotated_pair(q + a.d, i, a.rd, a.rot, a.cs + (size_t)t * (a.rot / 2));
            out[a.R + 2 * i] = v.x;
            if (a.R + 2 * i + 1 < a.RP) out[a.R + 2 * i + 1] = v.y;
        }
    }
}

// Any element type and size: a workgroup takes one query head of a token over one of n_split runs of keys, LAT_RUN at a
// time, with a running maximum; part[t, h, split] = {m, l, o[R]}, unnormalised.
constexpr int LAT_RUN = 64, LAT_MAX_SPLIT = 64, LAT_MAX_R = 2048;

template <class E>
__global__ __launch_bounds__(256) void latent_attention_any(LatentLayer a, const float *__restrict__ qx, int n_split, float *__restrict__ part) {
    using T = typename E::T;
    extern __shared__ float lsm[];  // q [RP], scores [LAT_RUN]
    float *qs = lsm, *sc = lsm + a.RP;
    const int split = blockIdx.x, h = blockIdx.y, t = blockIdx.z, tid = threadIdx.x, key = tid >> 2, sub = tid & 3;
    const int n = a.pos0 + t + 1, per = ((n + LAT_RUN - 1) / LAT_RUN + n_split - 1) / n_split * LAT_RUN;
    const int lo = split * per, hi = min(n, lo + per);
    const float *q = qx + ((size_t)t * a.H + h) * a.RP;
    for (int c = tid; c < a.RP; c += 256) qs[c] = q[c];
    float m = -INFINITY, l = 0.0f, acc[LAT_MAX_R / 256] = {};
    __syncthreads();
    for (int j0 = lo; j0 < hi; j0 += LAT_RUN) {
        const int nj = min(LAT_RUN, hi - j0);
        const uint8_t *kr = (const uint8_t *)((const T *)a.cache + (size_t)(j0 + min(key, nj - 1)) * a.RP);
        float s = 0.0f;
        for (int c = sub * E::CH; c < a.RP; c += 4 * E::CH) {
            float kv[E::CH];
            E::widen(chunk_of<E>(kr, c), kv);
#pragma unroll
            for (int i = 0; i < E::CH; i++) s = fmaf(qs[c + i], kv[i], s);
        }
        s += dpp_f<0xB1>(s);
        s += dpp_f<0x4E>(s);
        if (sub == 0) sc[key] = key < nj ? s * a.scale : -INFINITY;
        __syncthreads();
        const float v = sc[tid & 63], mn = fmaxf(m, wave_max(v)), e = expf(v - mn), keep = expf(m - mn);  // (every wave for itself)
        l = fmaf(l, keep, wave_sum(e));
        m = mn;
        __syncthreads();
        if (tid < 64) sc[tid] = e;
        __syncthreads();
#pragma unroll
        for (int i = 0; i < LAT_MAX_R / 256; i++) {
            const int c = tid + 256 * i;
            if (c >= a.R) break;
            float o = acc[i] * keep;
            for (int j = 0; j < nj; j++) o = fmaf(sc[j], (float)((const T *)a.cache)[(size_t)(j0 + j) * a.RP + c], o);
            acc[i] = o;
        }
        __syncthreads();
    }
    float *po = part + (((size_t)t * a.H + h) * n_split + split) * (a.R + 2);
#pragma unroll
    for (int i = 0; i < LAT_MAX_R / 256; i++)
        if (tid + 256 * i < a.R) po[2 + tid + 256 * i] = acc[i];
    if (tid == 0) po[0] = m, po[1] = l;
}

// The runs of a (token, head) merged, with the sink: olat[t, h] = sum_i f_i o_i / (sum_i f_i l_i + exp(sink - m)).  grid
// (T H, runs of 256 columns).
static __global__ __launch_bounds__(256) void latent_merge(const float *__restrict__ part, const float *__restrict__ sink, int H, int R,
                                                           int n_split, float *__restrict__ olat) {
    __shared__ float f[LAT_MAX_SPLIT], inv;
    const float *p = part + (size_t)blockIdx.x * n_split * (R + 2);
    if (threadIdx.x < 64) {
        const int i = threadIdx.x;
        const float mi = i < n_split ? p[(size_t)i * (R + 2)] : -INFINITY, li = i < n_split ? p[(size_t)i * (R + 2) + 1] : 0.0f;
        const float M = wave_max(mi), fi = mi == -INFINITY ? 0.0f : expf(mi - M);  // (a run without keys)
        float L = wave_sum(fi * li);
        if (sink) L += expf(sink[blockIdx.x % H] - M);
        if (i < LAT_MAX_SPLIT) f[i] = fi;
        if (i == 0) inv = 1.0f / L;
    }
    __syncthreads();
    const int c = (int)blockIdx.y * 256 + (int)threadIdx.x;
    if (c >= R) return;
    float v = 0.0f;
#pragma unroll 8
    for (int i = 0; i < n_split; i++) v = fmaf(p[(size_t)i * (R + 2) + 2 + c], f[i], v);
    olat[(size_t)blockIdx.x * R + c] = v * inv;
}

// out[t, h dv + j] = sigmoid(gate) (W_uv[h dv + j, :] . olat[t, h]): a wave takes four rows; grid (runs of 16 rows, heads, tokens).
template <class E>
__global__ __launch_bounds__(256) void latent_values(LatentLayer a, const float *__restrict__ olat, const uint8_t *__restrict__ Wuv,
                                                     size_t pitch, float *__restrict__ out) {
    const int h = blockIdx.y, t = blockIdx.z, lane = threadIdx.x & 63, j0 = ((int)blockIdx.x * 4 + ((int)threadIdx.x >> 6)) * 4;
    if (j0 >= a.dv) return;
    const float *x = olat + ((size_t)t * a.H + h) * a.R;
    float acc[4] = {};
    for (int c = lane * E::CH; c < a.R; c += 64 * E::CH) {
        float xv[E::CH];
        load_acts<E::CH>(x, c, a.R, xv);
#pragma unroll
        for (int r = 0; r < 4; r++) {
            float w[E::CH];
            E::widen(chunk_of<E>(Wuv + (size_t)(h * a.dv + min(j0 + r, a.dv - 1)) * pitch, c), w);
#pragma unroll
            for (int i = 0; i < E::CH; i++) acc[r] = fmaf(w[i], xv[i], acc[r]);
        }
    }
#pragma unroll
    for (int r = 0; r < 4; r++) {
        const float v = wave_sum(acc[r]);
        if (lane == r && j0 + r < a.dv) {
            const int col = h * a.dv + j0 + r;
            out[(size_t)t * a.H * a.dv + col] = v * sigmoid_of(a.gate[(size_t)t * a.ld + col]);
        }
    }
}

// ---- long steps ----

// Keys and values per head out of kv [n][H d + H dv] = [W_uk c | W_uv c]: kc [H][n][DP] = [unrotated | the row's rotated
// part], vc [H][n][DVP], zeros behind.  One workgroup a (key, run of heads).
template <class E>
__global__ __launch_bounds__(256) void latent_expand(LatentLayer a, const float *__restrict__ kv, int n, int DP, int DVP,
                                                     typename E::T *__restrict__ kc, typename E::T *__restrict__ vc) {
    using T = typename E::T;
    const int j = blockIdx.x;
    const float *row = kv + (size_t)j * a.H * (a.d + a.dv);
    const T *rot = (const T *)a.cache + (size_t)j * a.RP + a.R;
    for (int e = (int)blockIdx.y * 256 + (int)threadIdx.x; e < a.H * (DP + DVP); e += 256 * (int)gridDim.y) {
        const int h = e / (DP + DVP), c = e % (DP + DVP), cv = c - DP;
        if (c < DP) kc[((size_t)h * n + j) * DP + c] = c < a.d ? (T)row[h * a.d + c] : c < a.d + a.rd ? rot[c - a.d] : (T)0.0f;
        else vc[((size_t)h * n + j) * DVP + cv] = cv < a.dv ? (T)row[(size_t)a.H * a.d + h * a.dv + cv] : (T)0.0f;
    }
}

// The step's queries [T][H][DP], the rotated part turned.
template <class E>
__global__ __launch_bounds__(256) void latent_queries(LatentLayer a, int DP, typename E::T *__restrict__ qe) {
    using T = typename E::T;
    const int t = blockIdx.x, qd = a.d + a.rd;
    const float *row = a.q + (size_t)t * a.H * qd;
    const float2 *cs = a.cs + (size_t)t * (a.rot / 2);
    for (int e = threadIdx.x; e < a.H * DP; e += 256) {
        const int h = e / DP, c = e % DP;
        float v = 0.0f;
        if (c < a.d) {
            v = row[h * qd + c];
        } else if (c < qd) {
            const float2 p = rotated_pair(row + h * qd + a.d, (c - a.d) / 2, a.rd, a.rot, cs);
            v = (c - a.d) & 1 ? p.y : p.x;
        }
        qe[((size_t)t * a.H + h) * DP + c] = (T)v;
    }
}

}  // namespace jq
