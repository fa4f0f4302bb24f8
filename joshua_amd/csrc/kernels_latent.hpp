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

// qx[t, h] = [W_uk[h]^T q | rotated q], RP numbers a row (zeros behind), in f32 or as the matrix cores take them: grid (column runs of 16 chunks, heads + 1, tokens);
// the workgroups of the row behind the last head store the token's cache row.
template <class E, class O>
__global__ __launch_bounds__(256) void latent_absorb(LatentLayer a, const uint8_t *__restrict__ Wuk, size_t pitch, O *__restrict__ qx) {
    constexpr int CH = E::CH;
    __shared__ float part[16][16 * CH + 1], red[4];
    const int h = blockIdx.y, t = blockIdx.z, tid = threadIdx.x;
    if (h == a.H) {
        if (blockIdx.x == 0) latent_store_row<E>(a, t, red);
        return;
    }
    const float *q = a.q + ((size_t)t * a.H + h) * (a.d + a.rd);
    O *out = qx + ((size_t)t * a.H + h) * a.RP;
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
        out[c0 + tid] = (O)v;
    }
    if (blockIdx.x == 0) {
        for (int i = tid; i < (a.RP - a.R + 1) / 2; i += 256) {
            const float2 v = rotated_pair(q + a.d, i, a.rd, a.rot, a.cs + (size_t)t * (a.rot / 2));
            out[a.R + 2 * i] = (O)v.x;
            if (a.R + 2 * i + 1 < a.RP) out[a.R + 2 * i + 1] = (O)v.y;
        }
    }
}

// Any element type and size: a workgroup takes one query head of a token over one of n_split runs of keys, LAT_RUN at a
// time, with a running maximum; part[t, h, split] = {m, l, -, -, o[R]}, unnormalised.
constexpr int LAT_RUN = 64, LAT_MAX_SPLIT = 64, LAT_MAX_R = 2048;
__host__ __device__ inline int latent_part_width(int R) { return 4 + (R + 3) / 4 * 4; }

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
    float *po = part + (((size_t)t * a.H + h) * n_split + split) * latent_part_width(a.R);
#pragma unroll
    for (int i = 0; i < LAT_MAX_R / 256; i++)
        if (tid + 256 * i < a.R) po[4 + tid + 256 * i] = acc[i];
    if (tid == 0) po[0] = m, po[1] = l;
}

// The same in bf16 on the matrix cores: a workgroup takes 16 query heads of a token over a run of keys, 64 at a time.
//   scores  S^T = K Q^T: a wave's 16 keys and the heads' queries straight from memory, the first KF fragments of a row kept
//   softmax 16 threads a head, running maximum and sum; p goes on as the sum of two bf16 numbers
//   sums    O^T += C^T P^T: the cache rows' columns, 64 a wave at a time, transposed through LDS
// NB: runs of 256 latent columns.
constexpr int LATM_SROW = 68, LATM_PROW = 144;  // floats, bytes

template <int NB>
__global__ __launch_bounds__(256, 1) void latent_attention_mfma(LatentLayer a, const __bf16 *__restrict__ qx, int n_split, float *__restrict__ part) {
    constexpr int KF = 18;
    __shared__ __attribute__((aligned(16))) uint8_t ph[16 * LATM_PROW], pl[16 * LATM_PROW], stage[4 * 64 * TILE_COL];
    __shared__ __attribute__((aligned(16))) float sc[16 * LATM_SROW];
    __shared__ float al[16];
    const int split = blockIdx.x, h0 = 16 * (int)blockIdx.y, t = blockIdx.z, tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), l16 = lane & 15, g = lane >> 4;
    const int n = a.pos0 + t + 1, per = ((n + LAT_RUN - 1) / LAT_RUN + n_split - 1) / n_split * LAT_RUN;
    const int lo = split * per, hi = min(n, lo + per);
    const __bf16 *cache = (const __bf16 *)a.cache;
    // this wave's 16 keys of a tile, the first KF fragments of a row: on their way since before they are needed
    u32x4 kf[KF], qf[KF];
    auto fetch_keys = [&](int j0) __attribute__((always_inline)) {
        const __bf16 *kr = cache + (size_t)min(j0 + 16 * wave + l16, hi - 1) * a.RP + 8 * g;
#pragma unroll
        for (int i = 0; i < KF; i++)
            if (32 * i < a.RP) kf[i] = *(const u32x4 *)(kr + 32 * i);
    };
    // rows of a tile for the sums: tokens 2 pair, 2 pair + 1 and columns 8 c .. 8 c + 7 of this wave's 64
    const int uc = lane >> 3 & 7;
    u32x4 ra[NB][4], rb[NB][4];
    auto fetch_columns = [&](int j0) __attribute__((always_inline)) {
#pragma unroll
        for (int b = 0; b < NB; b++) {
            const int c0 = 256 * b + 64 * wave + 8 * uc;
            const __bf16 *base = cache + (c0 < a.RP ? c0 : 0);
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int j = j0 + 2 * ((lane & 7) + 8 * i);
                ra[b][i] = *(const u32x4 *)(base + (size_t)min(j, hi - 1) * a.RP);
                rb[b][i] = *(const u32x4 *)(base + (size_t)min(j + 1, hi - 1) * a.RP);
            }
        }
    };
    const __bf16 *qr = qx + ((size_t)t * a.H + min(h0 + l16, a.H - 1)) * a.RP + 8 * g;
    if (lo < hi) {
        fetch_keys(lo);
#pragma unroll
        for (int i = 0; i < KF; i++)
            if (32 * i < a.RP) qf[i] = *(const u32x4 *)(qr + 32 * i);
        fetch_columns(lo);
    }
    f32x4 o[NB][4];
#pragma unroll
    for (int b = 0; b < NB; b++)
#pragma unroll
        for (int i = 0; i < 4; i++) o[b][i] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.0f;  // of head tid / 16, the same in its 16 threads
    uint8_t *mine = stage + wave * 64 * TILE_COL;
    for (int j0 = lo; j0 < hi; j0 += LAT_RUN) {
        const int nj = min(LAT_RUN, hi - j0);
        f32x4 st{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < KF; i++)
            if (32 * i < a.RP) st = ElemBf16::mma(kf[i], qf[i], st);
        const __bf16 *kr = cache + (size_t)min(j0 + 16 * wave + l16, hi - 1) * a.RP + 8 * g;
        for (int c = 32 * KF; c < a.RP; c += 32)
            st = ElemBf16::mma(*(const u32x4 *)(kr + c), *(const u32x4 *)(qr + c), st);
        if (j0 + LAT_RUN < hi) fetch_keys(j0 + LAT_RUN);
        *(f32x4 *)(sc + l16 * LATM_SROW + 16 * wave + 4 * g) = st;
        __syncthreads();
        {
            const int hd = tid >> 4, k = 4 * (tid & 15);
            f32x4 s = *(const f32x4 *)(sc + hd * LATM_SROW + k), p;
#pragma unroll
            for (int r = 0; r < 4; r++) s[r] = k + r < nj ? s[r] * a.scale : -INFINITY;
            const float mn = fmaxf(m, max_row16(fmaxf(fmaxf(s[0], s[1]), fmaxf(s[2], s[3]))));  // (key j0 is there: finite)
#pragma unroll
            for (int r = 0; r < 4; r++) p[r] = expf(s[r] - mn);
            const float keep = expf(m - mn);
            l = fmaf(l, keep, sum_row16((p[0] + p[1]) + (p[2] + p[3])));
            m = mn;
            const bf16x4 hi4 = __builtin_convertvector(p, bf16x4), lo4 = __builtin_convertvector(p - __builtin_convertvector(hi4, f32x4), bf16x4);
            *(uint2 *)(ph + hd * LATM_PROW + 2 * k) = __builtin_bit_cast(uint2, hi4);
            *(uint2 *)(pl + hd * LATM_PROW + 2 * k) = __builtin_bit_cast(uint2, lo4);
            if ((tid & 15) == 0) al[hd] = keep;
        }
#pragma unroll
        for (int b = 0; b < NB; b++) {
            __syncthreads();  // p is there; and the fragments of the columns before are read
#pragma unroll
            for (int i = 0; i < 4; i++) tile_put(mine, uc, (lane & 7) + 8 * i, ra[b][i], rb[b][i]);
            if (b + 1 == NB && j0 + LAT_RUN < hi) fetch_columns(j0 + LAT_RUN);
            __syncthreads();
            const float keep = al[l16];
#pragma unroll
            for (int i = 0; i < 4; i++)
#pragma unroll
                for (int r = 0; r < 4; r++) o[b][i][r] *= keep;
#pragma unroll
            for (int ks = 0; ks < 2; ks++) {
                const u32x4 fh = *(const u32x4 *)(ph + l16 * LATM_PROW + 64 * ks + 16 * g), fl = *(const u32x4 *)(pl + l16 * LATM_PROW + 64 * ks + 16 * g);
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    const u32x4 v = *(const u32x4 *)(mine + tile_chunk(16 * i + l16, 4 * ks + g));
                    o[b][i] = ElemBf16::mma(v, fh, o[b][i]);
                    o[b][i] = ElemBf16::mma(v, fl, o[b][i]);
                }
            }
        }
        __syncthreads();
    }
    const int pw = latent_part_width(a.R);
    if (h0 + l16 < a.H) {
        float *po = part + (((size_t)t * a.H + h0 + l16) * n_split + split) * pw + 4;
#pragma unroll
        for (int b = 0; b < NB; b++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int c = 256 * b + 64 * wave + 16 * i + 4 * g;
                if (4 + c < pw) *(f32x4 *)(po + c) = o[b][i];
            }
    }
    if ((tid & 15) == 0 && h0 + (tid >> 4) < a.H) {
        float *po = part + (((size_t)t * a.H + h0 + (tid >> 4)) * n_split + split) * pw;
        po[0] = m, po[1] = l;
    }
}

// The runs of a (token, head) merged, with the sink, o = sum_i f_i o_i / (sum_i f_i l_i + exp(sink - m)), then
// out[t, h dv + j] = sigmoid(gate) (W_uv[h dv + j, :] . o): a wave takes LAT_VROWS rows; grid (runs of 4 LAT_VROWS rows,
// heads, tokens).
constexpr int LAT_VROWS = 8;

// NS: runs whose numbers are asked for ahead (n_split of them at most matter).
template <class E, int NS>
__global__ __launch_bounds__(256) void latent_values(LatentLayer a, const float *__restrict__ part, int n_split, const uint8_t *__restrict__ Wuv,
                                                     size_t pitch, float *__restrict__ out) {
    __shared__ __attribute__((aligned(16))) float ol[LAT_MAX_R];
    __shared__ float f[LAT_MAX_SPLIT], total;
    const int h = blockIdx.y, t = blockIdx.z, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, pw = latent_part_width(a.R);
    const int j0 = ((int)blockIdx.x * 4 + wave) * LAT_VROWS;
    const float *p = part + ((size_t)t * a.H + h) * n_split * pw;
    const bool works = j0 < a.dv;  // (the wave agrees)
    // the rows' first pieces are on their way while the runs are merged
    u32x4 w0[LAT_VROWS];
    const uint8_t *rows[LAT_VROWS];
#pragma unroll
    for (int r = 0; r < LAT_VROWS; r++) {
        rows[r] = Wuv + (size_t)(h * a.dv + min(j0 + r, a.dv - 1)) * pitch;
        w0[r] = chunk_of<E>(rows[r], min(lane * E::CH, (a.R - 1) / E::CH * E::CH));
    }
    float first[2][NS];  // the first columns' sums of the first runs
#pragma unroll
    for (int j = 0; j < 2; j++)
#pragma unroll
        for (int i = 0; i < NS; i++) first[j][i] = p[(size_t)min(i, n_split - 1) * pw + 4 + min((int)threadIdx.x + 256 * j, a.R - 1)];
    const int my_col = h * a.dv + min(j0 + (lane & (LAT_VROWS - 1)), a.dv - 1);
    const float z = a.gate[(size_t)t * a.ld + my_col];
    if (wave == 0) {
        const float mi = lane < n_split ? p[(size_t)lane * pw] : -INFINITY, li = lane < n_split ? p[(size_t)lane * pw + 1] : 0.0f;
        const float M = wave_max(mi), fi = mi == -INFINITY ? 0.0f : expf(mi - M);  // (a run without keys)
        float L = wave_sum(fi * li);
        if (a.sink) L += expf(a.sink[h] - M);
        f[lane] = fi;
        if (lane == 0) total = L;
    }
    __syncthreads();
    const float inv = 1.0f / total;
#pragma unroll
    for (int j = 0; j < 2; j++) {
        const int c = (int)threadIdx.x + 256 * j;
        float v = 0.0f;
#pragma unroll
        for (int i = 0; i < NS; i++)
            if (i < n_split) v = fmaf(first[j][i], f[i], v);
        if (c < a.R) ol[c] = v * inv;
    }
    for (int c = (int)threadIdx.x + 512; c < a.R; c += 256) {
        float v = 0.0f;
#pragma unroll 16
        for (int i = 0; i < n_split; i++) v = fmaf(p[(size_t)i * pw + 4 + c], f[i], v);
        ol[c] = v * inv;
    }
    __syncthreads();
    if (!works) return;
    float acc[LAT_VROWS] = {};
    for (int c = lane * E::CH; c < a.R; c += 64 * E::CH) {
        u32x4 w[LAT_VROWS];
#pragma unroll
        for (int r = 0; r < LAT_VROWS; r++) w[r] = c < 64 * E::CH ? w0[r] : chunk_of<E>(rows[r], c);
        float xv[E::CH];
        load_acts<E::CH>(ol, c, a.R, xv);
#pragma unroll
        for (int r = 0; r < LAT_VROWS; r++) {
            float wv[E::CH];
            E::widen(w[r], wv);
#pragma unroll
            for (int i = 0; i < E::CH; i++) acc[r] = fmaf(wv[i], xv[i], acc[r]);
        }
    }
#pragma unroll
    for (int r = 0; r < LAT_VROWS; r++) {
        const float v = wave_sum(acc[r]);
        if (lane == r && j0 + r < a.dv) out[(size_t)t * a.H * a.dv + my_col] = v * sigmoid_of(z);
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

// What products written by heads leave of those rows: the keys' rotated part and the zeros behind keys and values.
template <class E>
__global__ __launch_bounds__(256) void latent_rest_of_keys(LatentLayer a, int n, int DP, int DVP, typename E::T *__restrict__ kc,
                                                           typename E::T *__restrict__ vc) {
    using T = typename E::T;
    const int j = blockIdx.x, kr = DP - a.d, vr = DVP - a.dv;
    const T *rot = (const T *)a.cache + (size_t)j * a.RP + a.R;
    for (int e = threadIdx.x; e < a.H * kr; e += 256) {
        const int h = e / kr, c = e % kr;
        kc[((size_t)h * n + j) * DP + a.d + c] = c < a.rd ? rot[c] : (T)0.0f;
    }
    for (int e = threadIdx.x; e < a.H * vr; e += 256) vc[((size_t)(e / vr) * n + j) * DVP + a.dv + e % vr] = (T)0.0f;
}

// The step's queries [T][H][DP], the rotated part turned.
template <class E>
__global__ __launch_bounds__(256) void latent_queries(LatentLayer a, int DP, typename E::T *__restrict__ qe) {
    using T = typename E::T;
    typedef T T2 __attribute__((ext_vector_type(2)));
    typedef T T4 __attribute__((ext_vector_type(4)));
    const int t = blockIdx.x, qd = a.d + a.rd;
    const float *row = a.q + (size_t)t * a.H * qd;
    const float2 *cs = a.cs + (size_t)t * (a.rot / 2);
    if (((a.d | a.rd | a.rot) & 3) == 0) {
        for (int e = threadIdx.x; e < a.H * (DP / 4); e += 256) {
            const int h = e / (DP / 4), c = 4 * (e % (DP / 4)), i = c - a.d;
            f32x4 v = *(const f32x4 *)(row + h * qd + min(c, qd - 4));
            if (i >= 0 && i < a.rot) {
                const f32x4 r = *(const f32x4 *)(cs + i / 2);
                v = f32x4{v[0] * r[0] - v[1] * r[1], v[1] * r[0] + v[0] * r[1], v[2] * r[2] - v[3] * r[3], v[3] * r[2] + v[2] * r[3]};
            }
            if (c >= qd) v = f32x4{0.f, 0.f, 0.f, 0.f};
            *(T4 *)(qe + ((size_t)t * a.H + h) * DP + c) = T4{(T)v[0], (T)v[1], (T)v[2], (T)v[3]};
        }
        return;
    }
    for (int e = threadIdx.x; e < a.H * (DP / 2); e += 256) {
        const int h = e / (DP / 2), c0 = 2 * (e % (DP / 2));
        const float *q = row + h * qd;
        auto element = [&](int c) {
            if (c < a.d) return q[c];
            if (c >= qd) return 0.0f;
            const float2 p = rotated_pair(q + a.d, (c - a.d) / 2, a.rd, a.rot, cs);
            return (c - a.d) & 1 ? p.y : p.x;
        };
        *(T2 *)(qe + ((size_t)t * a.H + h) * DP + c0) = T2{(T)element(c0), (T)element(c0 + 1)};
    }
}

}  // namespace jq
