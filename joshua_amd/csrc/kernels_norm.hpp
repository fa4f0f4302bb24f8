// The residual stream of decoders that normalise in front of and behind a sublayer: x + mult * norm(y), then the norm
// of the result for the next sublayer, f32 throughout, one workgroup of 256 a row.
#pragma once
#include "kernels_graph.hpp"

namespace jq {

struct ResidualNorm {
    const float *x;                    // the residual stream, rows `width` apart
    const float *y;                    // the sublayer's result to add, or null
    const float *post_w, *post_b;      // the norm on y (post_w null: y as it is)
    float mult;
    const float *pre_w, *pre_b;        // the norm that makes h
    float eps;
    int rms;                           // both norms: 1 root mean square, 0 mean and variance (with bias)
    int width;
    float *x_out;                      // may be x, except where other workgroups read the row
    float *h_out;                      // or null
};

// sum over the workgroup of 256, in every thread; `red` is not used again before another barrier
__device__ __forceinline__ float sum256(float v, float *red) {
    v = wave_sum(v);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}

// One norm over the row held as v[i] at column threadIdx.x + 256 i (0 past the width): mean and 1 / deviation.
template <int NV>
__device__ __forceinline__ void row_stats(const float (&v)[NV], int width, float eps, int rms, float *red, float *mean, float *inv) {
    float mu = 0.0f;
    if (!rms) {
        float s = 0.0f;
#pragma unroll
        for (int i = 0; i < NV; i++) s += v[i];
        mu = sum256(s, red) / (float)width;
    }
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < NV; i++) {
        const float d = (int)threadIdx.x + 256 * i < width ? v[i] - mu : 0.0f;
        ss = fmaf(d, d, ss);
    }
    *mean = mu;
    *inv = 1.0f / sqrtf(sum256(ss, red + 4) / (float)width + eps);
}

// Row `row` of the update; the normed row goes to `h` (LDS or global), and with `store` x and h to x_out and h_out.
template <int NV>
__device__ __forceinline__ void residual_norm_row(const ResidualNorm &a, size_t row, float *h, bool store) {
    __shared__ float red[16];  // a row of four for each of the sums
    const float *xr = a.x + row * a.width;
    float x[NV], mean, inv;
    const int c0 = threadIdx.x;
#pragma unroll
    for (int i = 0; i < NV; i++) x[i] = c0 + 256 * i < a.width ? xr[c0 + 256 * i] : 0.0f;
    if (a.y) {
        const float *yr = a.y + row * a.width;
        float y[NV];
#pragma unroll
        for (int i = 0; i < NV; i++) y[i] = c0 + 256 * i < a.width ? yr[c0 + 256 * i] : 0.0f;
        if (a.post_w) {
            row_stats<NV>(y, a.width, a.eps, a.rms, red, &mean, &inv);
#pragma unroll
            for (int i = 0; i < NV; i++) {
                const int c = c0 + 256 * i;
                if (c < a.width) y[i] = fmaf((y[i] - mean) * inv, a.post_w[c], a.post_b ? a.post_b[c] : 0.0f);
            }
        }
#pragma unroll
        for (int i = 0; i < NV; i++) x[i] = fmaf(a.mult, y[i], x[i]);
    }
    row_stats<NV>(x, a.width, a.eps, a.rms, red + 8, &mean, &inv);
#pragma unroll
    for (int i = 0; i < NV; i++) {
        const int c = c0 + 256 * i;
        if (c >= a.width) continue;
        const float v = fmaf((x[i] - mean) * inv, a.pre_w[c], a.pre_b ? a.pre_b[c] : 0.0f);
        if (h) h[c] = v;
        if (store) {
            if (a.x_out) a.x_out[row * a.width + c] = x[i];
            if (a.h_out) a.h_out[row * a.width + c] = v;
        }
    }
}

// The update of many rows: x in place, h in f32 (h_out) and / or in the products' element type (he, rows `stride`
// apart, zeros behind the width).  `at`: the rows to take (x_out is then left alone), or null for rows 0, 1, ..
template <class E, int NV>
__global__ __launch_bounds__(256) void residual_norm_rows(ResidualNorm a, typename E::T *__restrict__ he, size_t stride,
                                                          const uint32_t *__restrict__ at) {
    extern __shared__ float hrow[];  // [width] when he is given
    const size_t row = at ? at[blockIdx.x] : blockIdx.x;
    if (at) {  // rows of the stream gathered into the first rows of h
        ResidualNorm b = a;
        b.x_out = nullptr, b.h_out = nullptr;
        residual_norm_row<NV>(b, row, he ? hrow : a.h_out + (size_t)blockIdx.x * a.width, false);
    } else {
        residual_norm_row<NV>(a, row, he ? hrow : nullptr, true);
    }
    if (!he) return;
    __syncthreads();
    typename E::T *out = he + (size_t)blockIdx.x * stride;
    for (int c = threadIdx.x; c < (int)stride; c += 256) out[c] = (typename E::T)(c < a.width ? hrow[c] : 0.0f);
}

}  // namespace jq
