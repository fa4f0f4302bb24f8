// The residual stream of decoders that normalise in front of and behind a sublayer: x + mult * norm(y), then the norm
// of the result for the next sublayer, f32 throughout, one workgroup of BT threads a row.
#pragma once
#include "kernels_graph.hpp"

namespace jq {

struct ResidualNorm {
    const float *x;                    // the residual stream
    const float *y;                    // the sublayer's result to add, or null
    const float *post_w, *post_b;      // the norm on y (post_w null: y as it is)
    float mult;
    const float *pre_w, *pre_b;        // the norm that makes h
    float eps;
    int rms;                           // both norms: 1 root mean square, 0 mean and variance (with bias)
    int width;
    size_t ldx;                        // x: from a row to the next (0: width)
    float *x_out;                      // may be x, except where other workgroups read the row
    float *h_out;                      // or null
};

// sum over the workgroup of BT, in every thread; `red` [BT / 64] is not used again before another barrier
template <int BT>
__device__ __forceinline__ float sum_block(float v, float *red) {
    v = wave_sum(v);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = 0.0f;
#pragma unroll
    for (int i = 0; i < BT / 64; i++) s += red[i];
    return s;
}

// Element i of a thread's share of a row: four columns side by side, every 4 BT.
template <int BT>
__device__ __forceinline__ int norm_col(int i) { return 4 * (int)threadIdx.x + 4 * BT * (i / 4) + i % 4; }

// The thread's share of a row; columns past the width are zero.  Every load is issued whatever the width (past it, from
// the row's end), so that the loads of a row's vectors travel together.
template <int NV, int BT>
__device__ __forceinline__ void load_row(const float *__restrict__ p, int width, float (&v)[NV]) {
    if ((width & 3) == 0) {
#pragma unroll
        for (int i = 0; i < NV; i += 4) {
            const float4 q = *(const float4 *)(p + min(norm_col<BT>(i), width - 4));
            v[i] = q.x, v[i + 1] = q.y, v[i + 2] = q.z, v[i + 3] = q.w;
        }
    } else {
#pragma unroll
        for (int i = 0; i < NV; i++) v[i] = p[min(norm_col<BT>(i), width - 1)];
    }
#pragma unroll
    for (int i = 0; i < NV; i++) v[i] = norm_col<BT>(i) < width ? v[i] : 0.0f;
}

template <int NV, int BT>
__device__ __forceinline__ void store_row(float *__restrict__ p, int width, const float (&v)[NV]) {
    if ((width & 3) == 0) {
#pragma unroll
        for (int i = 0; i < NV; i += 4)
            if (norm_col<BT>(i) < width) *(float4 *)(p + norm_col<BT>(i)) = float4{v[i], v[i + 1], v[i + 2], v[i + 3]};
    } else {
#pragma unroll
        for (int i = 0; i < NV; i++)
            if (norm_col<BT>(i) < width) p[norm_col<BT>(i)] = v[i];
    }
}

// One norm over the row held as v (0 past the width): mean and 1 / deviation.
template <int NV, int BT>
__device__ __forceinline__ void row_stats(const float (&v)[NV], int width, float eps, int rms, float *red, float *mean, float *inv) {
    float mu = 0.0f;
    if (!rms) {
        float s = 0.0f;
#pragma unroll
        for (int i = 0; i < NV; i++) s += v[i];
        mu = sum_block<BT>(s, red) / (float)width;
    }
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < NV; i++) {
        const float d = norm_col<BT>(i) < width ? v[i] - mu : 0.0f;
        ss = fmaf(d, d, ss);
    }
    *mean = mu;
    *inv = 1.0f / sqrtf(sum_block<BT>(ss, red + BT / 64) / (float)width + eps);
}

// The update of one row by a workgroup; x ends as this thread's share of the normed row.  With `store` the stream goes to
// x_out and the normed row to h_out.  The norms' vectors are asked for together with the row: a single row's time is its
// round trips to memory.
template <int NV, int BT>
__device__ __forceinline__ void residual_norm_row(const ResidualNorm &a, float (&x)[NV], bool store) {
    __shared__ float red[4 * (BT / 64)];  // a part for each of the sums
    const int w = a.width;
    float g[NV], b[NV], mean, inv;
    load_row<NV, BT>(a.x, w, x);
    if (a.y) {
        float y[NV], pg[NV], pb[NV];
        load_row<NV, BT>(a.y, w, y);
        if (a.post_w) load_row<NV, BT>(a.post_w, w, pg);
        if (a.post_w && a.post_b) load_row<NV, BT>(a.post_b, w, pb);
        load_row<NV, BT>(a.pre_w, w, g);
        if (a.pre_b) load_row<NV, BT>(a.pre_b, w, b);
        if (a.post_w) {
            row_stats<NV, BT>(y, w, a.eps, a.rms, red, &mean, &inv);
#pragma unroll
            for (int i = 0; i < NV; i++) y[i] = norm_col<BT>(i) < w ? fmaf((y[i] - mean) * inv, pg[i], a.post_b ? pb[i] : 0.0f) : 0.0f;
        }
#pragma unroll
        for (int i = 0; i < NV; i++) x[i] = fmaf(a.mult, y[i], x[i]);
    } else {
        load_row<NV, BT>(a.pre_w, w, g);
        if (a.pre_b) load_row<NV, BT>(a.pre_b, w, b);
    }
    if (store && a.x_out) store_row<NV, BT>(a.x_out, w, x);
    row_stats<NV, BT>(x, w, a.eps, a.rms, red + 2 * (BT / 64), &mean, &inv);
#pragma unroll
    for (int i = 0; i < NV; i++) x[i] = fmaf((x[i] - mean) * inv, g[i], a.pre_b ? b[i] : 0.0f);
    if (store && a.h_out) store_row<NV, BT>(a.h_out, w, x);
}

// The update of many rows, a workgroup a row: x in place, h in f32 (h_out) and / or in the products' element type (he, rows
// `stride` apart, zeros behind the width).  `at`: the rows to take, into the first rows of h (x_out is then left alone), or
// null for rows 0, 1, ..  A thread has columns BT apart, and the norms' vectors are read as they are needed: what counts here
// is how many rows are under way at once, that is registers.
template <class E, int NV, int BT>
__global__ __launch_bounds__(BT) void residual_norm_rows(ResidualNorm a, typename E::T *__restrict__ he, size_t stride,
                                                         const uint32_t *__restrict__ at) {
    using T = typename E::T;
    constexpr int NW = BT / 64;
    __shared__ float red[4 * NW];
    const int w = a.width, c0 = threadIdx.x;
    const size_t row = at ? at[blockIdx.x] : blockIdx.x;
    const float *xr = a.x + row * (a.ldx ? a.ldx : (size_t)w);
    float x[NV];
    auto stats = [&](const float (&v)[NV], float *r, float *mean, float *inv) __attribute__((always_inline)) {
        float mu = 0.0f, ss = 0.0f;
        if (!a.rms) {
            float s = 0.0f;
#pragma unroll
            for (int i = 0; i < NV; i++) s += v[i];
            mu = sum_block<BT>(s, r) / (float)w;
        }
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const float d = c0 + BT * i < w ? v[i] - mu : 0.0f;
            ss = fmaf(d, d, ss);
        }
        *mean = mu, *inv = 1.0f / sqrtf(sum_block<BT>(ss, r + NW) / (float)w + a.eps);
    };
#pragma unroll
    for (int i = 0; i < NV; i++) x[i] = c0 + BT * i < w ? xr[c0 + BT * i] : 0.0f;
    float mean, inv;
    if (a.y) {
        const float *yr = a.y + row * w;
        float y[NV];
#pragma unroll
        for (int i = 0; i < NV; i++) y[i] = c0 + BT * i < w ? yr[c0 + BT * i] : 0.0f;
        if (a.post_w) {
            stats(y, red, &mean, &inv);
#pragma unroll
            for (int i = 0; i < NV; i++) {
                const int c = c0 + BT * i;
                if (c < w) y[i] = fmaf((y[i] - mean) * inv, a.post_w[c], a.post_b ? a.post_b[c] : 0.0f);
            }
        }
#pragma unroll
        for (int i = 0; i < NV; i++) x[i] = fmaf(a.mult, y[i], x[i]);
    }
    stats(x, red + 2 * NW, &mean, &inv);
    float *xo = at ? nullptr : a.x_out, *ho = a.h_out ? a.h_out + (size_t)blockIdx.x * w : nullptr;
    T *eo = he ? he + (size_t)blockIdx.x * stride : nullptr;
#pragma unroll
    for (int i = 0; i < NV; i++) {
        const int c = c0 + BT * i;
        if (c < w) {
            const float v = fmaf((x[i] - mean) * inv, a.pre_w[c], a.pre_b ? a.pre_b[c] : 0.0f);
            if (xo) xo[row * w + c] = x[i];
            if (ho) ho[c] = v;
            if (eo) eo[c] = (T)v;
        } else if (eo && c < (int)stride) {
            eo[c] = (T)0.0f;
        }
    }
}

}  // namespace jq
