// Products with plain weight rows, BF16 or F32: a GEMV for up to 8 activation rows (f32 activations), a tiled GEMM on
// the matrix cores for more (activations in the weights' type), both also for the gated pair of a feed-forward block
// and for grouped experts.  Weight rows are padded with zeros to whole runs of 64 elements, so a row is read in
// 16-byte chunks without a tail.
#pragma once
#include "kernels_norm.hpp"

namespace jq {

typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));

// Element types: CH elements to a chunk of 16 bytes; mma multiplies two fragments of 16 rows x 4 chunks (lane l:
// row l % 16, chunk l / 16) into a 16 x 16 tile (lane l: rows 4 (l / 16) + r of the first, column l % 16 = row of
// the second operand), f32 accumulation.
struct ElemBf16 {
    using T = __bf16;
    static constexpr int CH = 8, BYTES = 2;
    static __device__ __forceinline__ void widen(const u32x4 &raw, float (&f)[CH]) {
#pragma unroll
        for (int i = 0; i < 4; i++) {
            f[2 * i] = __builtin_bit_cast(float, raw[i] << 16);
            f[2 * i + 1] = __builtin_bit_cast(float, raw[i] & 0xFFFF0000u);
        }
    }
    static __device__ __forceinline__ f32x4 mma(const u32x4 &a, const u32x4 &b, const f32x4 &c) {
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
    }
};
struct ElemF32 {
    using T = float;
    static constexpr int CH = 4, BYTES = 4;
    static __device__ __forceinline__ void widen(const u32x4 &raw, float (&f)[CH]) {
        const f32x4 v = __builtin_bit_cast(f32x4, raw);
#pragma unroll
        for (int i = 0; i < 4; i++) f[i] = v[i];
    }
    // (element i of a chunk in step i: any order of the inner index serves, as long as both operands share it)
    static __device__ __forceinline__ f32x4 mma(const u32x4 &a, const u32x4 &b, f32x4 c) {
        const f32x4 av = __builtin_bit_cast(f32x4, a), bv = __builtin_bit_cast(f32x4, b);
#pragma unroll
        for (int i = 0; i < 4; i++) c = __builtin_amdgcn_mfma_f32_16x16x4f32(av[i], bv[i], c, 0, 0, 0);
        return c;
    }
};

// The gated unit of a feed-forward block: g sigmoid(alpha g) (u + shift), g and u clamped first.
struct GatedUnit {
    float limit, alpha, shift;  // limit INFINITY: no clamp
    __device__ __forceinline__ float operator()(float g, float u) const {
        g = g > limit ? limit : g;  // (comparisons: a NaN stays a NaN)
        u = u > limit ? limit : (u < -limit ? -limit : u);
        return g / (1.0f + expf(-alpha * g)) * (u + shift);
    }
};

template <class E>
__device__ __forceinline__ u32x4 chunk_of(const uint8_t *row, int c) {
    return *(const u32x4 *)(row + (size_t)c * E::BYTES);
}

// ---- GEMV -----------------------------------------------------------------------------------------

// CH activations from column c on; columns at and past k are zero.
template <int CH>
__device__ __forceinline__ void load_acts(const float *__restrict__ x, int c, int k, float (&f)[CH]) {
    if (c + CH <= k) {
#pragma unroll
        for (int i = 0; i < CH; i += 4) {
            const float4 v = ld<float4>((const uint8_t *)(x + c + i));
            f[i] = v.x, f[i + 1] = v.y, f[i + 2] = v.z, f[i + 3] = v.w;
        }
    } else {
#pragma unroll
        for (int i = 0; i < CH; i++) f[i] = c + i < k ? x[c + i] : 0.0f;
    }
}

// acc[m][r] += x[m] . rows[r] (m past the rows of x: the last one again) over this thread's chunks (a workgroup of 256
// shares the row), from pass `p0` on.
template <class E, int MT, int R>
__device__ __forceinline__ void gemv_accumulate(const uint8_t *const (&rows)[R], const float *__restrict__ x, size_t ldx, int rows_of_x,
                                                int k, float (&acc)[MT][R], int p0 = 0) {
    constexpr int STEP = 256 * E::CH;
#pragma unroll 2
    for (int c = (int)threadIdx.x * E::CH + p0 * STEP; c < k; c += STEP) {
        u32x4 w[R];
#pragma unroll
        for (int r = 0; r < R; r++) w[r] = chunk_of<E>(rows[r], c);
#pragma unroll
        for (int m = 0; m < MT; m++) {
            float xv[E::CH];
            load_acts<E::CH>(x + (MT > 1 ? min(m, rows_of_x - 1) : 0) * ldx, c, k, xv);
#pragma unroll
            for (int r = 0; r < R; r++) {
                float wv[E::CH];
                E::widen(w[r], wv);
#pragma unroll
                for (int i = 0; i < E::CH; i++) acc[m][r] = fmaf(wv[i], xv[i], acc[m][r]);
            }
        }
    }
}

// Sums of the four waves' accumulators; value v of the N belongs to thread v (others: undefined).
template <int N>
__device__ __forceinline__ float gemv_reduce(const float (&acc)[N], float (&red)[4][N]) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
#pragma unroll
    for (int i = 0; i < N; i++) {
        const float s = wave_sum(acc[i]);
        if (lane == 0) red[wave][i] = s;
    }
    __syncthreads();
    const int v = threadIdx.x;
    return v < N ? (red[0][v] + red[1][v]) + (red[2][v] + red[3][v]) : 0.0f;
}

// Y[m, n] = X[m, :] . W[n, :] for m < MT rows, four weight rows a workgroup.
template <class E, int MT>
__global__ __launch_bounds__(256) void dense_gemv(const uint8_t *__restrict__ W, size_t pitch, const float *__restrict__ X,
                                                  size_t ldx, float *__restrict__ Y, size_t ldy, int rows_of_x, int k, int n) {
    constexpr int R = 4;
    __shared__ float red[4][MT * R];
    const int r0 = R * (int)blockIdx.x;
    const uint8_t *rows[R];
#pragma unroll
    for (int r = 0; r < R; r++) rows[r] = W + (size_t)min(r0 + r, n - 1) * pitch;
    float acc[MT][R] = {};
    gemv_accumulate<E, MT, R>(rows, X, ldx, rows_of_x, k, acc);
    float flat[MT * R];
#pragma unroll
    for (int m = 0; m < MT; m++)
#pragma unroll
        for (int r = 0; r < R; r++) flat[m * R + r] = acc[m][r];
    const float y = gemv_reduce<MT * R>(flat, red);
    const int m = (int)threadIdx.x / R, r = (int)threadIdx.x % R;
    if (m < min(MT, rows_of_x) && r0 + r < n) Y[m * ldy + r0 + r] = y;
}

// Y[m, j] = gated(X[m] . Wg[j], X[m] . Wu[j]), two j a workgroup.
template <class E, int MT>
__global__ __launch_bounds__(256) void dense_gemv_gated(const uint8_t *__restrict__ Wg, const uint8_t *__restrict__ Wu,
                                                        size_t pitch, const float *__restrict__ X, size_t ldx,
                                                        float *__restrict__ Y, size_t ldy, int rows_of_x, int k, int n, GatedUnit act) {
    constexpr int R = 4;
    __shared__ float red[4][MT * R], sums[MT * R];
    const int j0 = 2 * (int)blockIdx.x;
    const uint8_t *rows[R];
#pragma unroll
    for (int r = 0; r < R; r++) rows[r] = (r & 1 ? Wu : Wg) + (size_t)min(j0 + (r >> 1), n - 1) * pitch;
    float acc[MT][R] = {};
    gemv_accumulate<E, MT, R>(rows, X, ldx, rows_of_x, k, acc);
    float flat[MT * R];
#pragma unroll
    for (int m = 0; m < MT; m++)
#pragma unroll
        for (int r = 0; r < R; r++) flat[m * R + r] = acc[m][r];
    const float s = gemv_reduce<MT * R>(flat, red);
    if (threadIdx.x < MT * R) sums[threadIdx.x] = s;
    __syncthreads();
    const int m = (int)threadIdx.x / 2, j = (int)threadIdx.x % 2;
    if (m < min(MT, rows_of_x) && j0 + j < n) Y[m * ldy + j0 + j] = act(sums[m * R + 2 * j], sums[m * R + 2 * j + 1]);
}

// The one-row products with the residual update and norm of `nm` in front: y = W h, or with GATED
// y = gated(Wg h, Wu h).  A workgroup makes the normed row h for itself (workgroup 0 stores it; few, large
// workgroups, since each reads the norm's vectors whole); then every wave takes pairs of weight rows (gated: the gate and the
// up row of a column) on its own, the first chunks of its first pair on their way since before the norm.
template <class E, int WAVES, int NV, bool GATED>
__global__ __launch_bounds__(64 * WAVES) void norm_gemv(const uint8_t *__restrict__ W, const uint8_t *__restrict__ Wu, size_t pitch,
                                                                  float *__restrict__ Y, int k, int n, GatedUnit act, ResidualNorm nm) {
    constexpr int R = 2, PER = GATED ? 1 : 2, STEP = 64 * E::CH, PRE = 4;
    extern __shared__ __attribute__((aligned(16))) float hrow[];  // [k]
    const int groups = (n + PER - 1) / PER, lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const uint8_t *rows[R];
    u32x4 pre[PRE][R];
    auto ask = [&](int grp) __attribute__((always_inline)) {
#pragma unroll
        for (int r = 0; r < R; r++) rows[r] = (GATED && r ? Wu : W) + (size_t)min(GATED ? grp : 2 * grp + r, n - 1) * pitch;
#pragma unroll
        for (int p = 0; p < PRE; p++) {  // (past the row: its last chunk, multiplied by nothing)
            const int c = min(lane * E::CH + p * STEP, (k - 1) / E::CH * E::CH);
#pragma unroll
            for (int r = 0; r < R; r++) pre[p][r] = chunk_of<E>(rows[r], c);
        }
    };
    auto multiply = [&](const u32x4 (&w)[R], int c, float (&acc)[R]) __attribute__((always_inline)) {
        float xv[E::CH];
        load_acts<E::CH>(hrow, c, k, xv);
#pragma unroll
        for (int r = 0; r < R; r++) {
            float wv[E::CH];
            E::widen(w[r], wv);
#pragma unroll
            for (int i = 0; i < E::CH; i++) acc[r] = fmaf(wv[i], xv[i], acc[r]);
        }
    };
    int grp = (int)blockIdx.x + (int)gridDim.x * wave;
    ask(min(grp, groups - 1));
    {
        float h[NV];
        residual_norm_row<NV, 64 * WAVES>(nm, h, blockIdx.x == 0);
        store_row<NV, 64 * WAVES>(hrow, k, h);
    }
    __syncthreads();
    for (; grp < groups; grp += (int)gridDim.x * WAVES) {
        float acc[R] = {};
#pragma unroll
        for (int p = 0; p < PRE; p++) {
            const int c = lane * E::CH + p * STEP;
            if (c < k) multiply(pre[p], c, acc);
        }
#pragma unroll 4
        for (int c = lane * E::CH + PRE * STEP; c < k; c += STEP) {
            u32x4 w[R];
#pragma unroll
            for (int r = 0; r < R; r++) w[r] = chunk_of<E>(rows[r], c);
            multiply(w, c, acc);
        }
        const int next = grp + (int)gridDim.x * WAVES;
        if (next < groups) ask(next);
#pragma unroll
        for (int r = 0; r < R; r++) acc[r] = wave_sum(acc[r]);
        if (GATED) {
            if (lane == 0) Y[grp] = act(acc[0], acc[1]);
        } else if (lane < R && 2 * grp + lane < n) {
            Y[2 * grp + lane] = lane ? acc[1] : acc[0];
        }
    }
}

// The shared expert beside a decode-sized call's pairs: rows pairs .. pairs + T - 1 of the gate|up grid.
struct SharedRows {
    const uint8_t *gate, *up;  // null: none
    int n;                     // its activations a token
    float *act;                // [T][n]
    const float *logit;        // token t's activations are multiplied by sigmoid(logit[t ld]); null: left alone
    size_t ld;
    int pairs;
    float limit;               // its own clamp
};

__device__ __forceinline__ float sigmoid_of(float z) { return 1.0f / (1.0f + expf(-z)); }

// The experts' gated pairs of a decode-sized call: blockIdx.y is the (token, slot) pair, four j a workgroup, every
// weight row read once a pair.  NE > 0: the workgroup's first wave runs the token's gating over the router's logits
// (moe_gate_topk_wave's arithmetic); the first workgroup of a token's first pair writes ids and weights for the
// down projection.  NE = 0: the ids are there.
template <class E, int NE>
__global__ __launch_bounds__(256) void moe_dense_gate_up(const uint8_t *const *__restrict__ Wg, const uint8_t *const *__restrict__ Wu,
                                                         size_t pitch, const float *__restrict__ X, size_t ldx,
                                                         float *__restrict__ Y, size_t ldy, int k, int n, int k_used,
                                                         const uint32_t *__restrict__ ids, GatedUnit act, MoeGateIn gi, SharedRows sh) {
    constexpr int R = 8;
    __shared__ float red[4][R], sums[R];
    __shared__ int expert;
    const bool shared = (int)blockIdx.y >= sh.pairs;  // (the workgroup agrees)
    const int pair = shared ? (int)blockIdx.y - sh.pairs : (int)blockIdx.y, t = shared ? pair : pair / k_used, slot = pair % k_used;
    if (shared) Y = sh.act, ldy = (size_t)sh.n, n = sh.n, act.limit = sh.limit;
    if (R / 2 * (int)blockIdx.x >= n) return;  // (the grid is as wide as the wider of the two)
    int e = 0;
    if (shared) {
    } else if constexpr (NE > 0) {
        if (threadIdx.x < 64) {
            int slot_e;
            moe_gate_topk_wave_body<NE>(t, gi.T, (int)threadIdx.x, gi.logits, gi.bias, gi.p, gi.ids, gi.wts, gi.pg,
                                        blockIdx.x == 0 && slot == 0, &slot_e);
            if ((int)threadIdx.x == slot) expert = slot_e;
        }
        __syncthreads();
        e = expert;
    } else {
        e = min((int)ids[pair], gi.p.E - 1);
    }
    e = __builtin_amdgcn_readfirstlane(e);
    const int j0 = (R / 2) * (int)blockIdx.x;
    const uint8_t *rows[R];
#pragma unroll
    for (int r = 0; r < R; r++)
        rows[r] = (shared ? (r & 1 ? sh.up : sh.gate) : (r & 1 ? Wu : Wg)[e]) + (size_t)min(j0 + (r >> 1), n - 1) * pitch;
    float acc[1][R] = {};
    gemv_accumulate<E, 1, R>(rows, X + (size_t)t * ldx, 0, 1, k, acc);
    const float s = gemv_reduce<R>(acc[0], red);
    if (threadIdx.x < R) sums[threadIdx.x] = s;
    __syncthreads();
    const int j = (int)threadIdx.x;
    if (j < R / 2 && j0 + j < n) {
        const float v = act(sums[2 * j], sums[2 * j + 1]);
        Y[(size_t)pair * ldy + j0 + j] = shared && sh.logit ? sigmoid_of(sh.logit[t * sh.ld]) * v : v;
    }
}

// A product that joins a sum of products: + W[n, :] . x[t, :].
struct SumRun {
    const uint8_t *W;   // null: none
    size_t pitch;
    const float *x;
    size_t ldx;
    int k;
};

// y[t, :] = sum over the token's slots of weight * (W_down[expert] act[pair]), plus two runs of their own (a shared
// expert's down projection, the mixer's output projection) and the row `add`: down projections and combine of a
// decode-sized call.  Four rows a workgroup; its threads share the (slot, chunk) list.
template <class E>
__global__ __launch_bounds__(256) void moe_dense_down(const uint8_t *const *__restrict__ Wd, size_t pitch,
                                                      const float *__restrict__ A, size_t lda, const uint32_t *__restrict__ ids,
                                                      const float *__restrict__ wts, float *y, int k, int n,
                                                      int k_used, int n_expert, SumRun run1, SumRun run2, const float *add) {
    constexpr int R = 4;
    __shared__ float red[4][R];
    const int t = blockIdx.y, r0 = R * (int)blockIdx.x;
    const int per = (k + E::CH - 1) / E::CH, total = per * k_used;
    const int per1 = run1.W ? (run1.k + E::CH - 1) / E::CH : 0, per2 = run2.W ? (run2.k + E::CH - 1) / E::CH : 0;
    float acc[R] = {};
#pragma unroll 2
    for (int i = threadIdx.x; i < total + per1 + per2; i += 256) {
        const uint8_t *base;
        const float *x;
        size_t pt = pitch;
        int c, kk = k;
        float wt = 1.0f;
        if (i < total) {
            const int slot = i / per, pair = t * k_used + slot;
            c = (i % per) * E::CH, base = Wd[min((int)ids[pair], n_expert - 1)], x = A + (size_t)pair * lda, wt = wts[pair];
        } else {
            const bool first = i < total + per1;
            c = (i - total - (first ? 0 : per1)) * E::CH, base = first ? run1.W : run2.W, pt = first ? run1.pitch : run2.pitch;
            x = first ? run1.x + t * run1.ldx : run2.x + t * run2.ldx, kk = first ? run1.k : run2.k;
        }
        u32x4 w[R];
#pragma unroll
        for (int r = 0; r < R; r++) w[r] = chunk_of<E>(base + (size_t)min(r0 + r, n - 1) * pt, c);
        float xv[E::CH];
        load_acts<E::CH>(x, c, kk, xv);
#pragma unroll
        for (int r = 0; r < R; r++) {
            float wv[E::CH], d = 0.0f;
            E::widen(w[r], wv);
#pragma unroll
            for (int j = 0; j < E::CH; j++) d = fmaf(wv[j], xv[j], d);
            acc[r] = fmaf(wt, d, acc[r]);
        }
    }
    const float s = gemv_reduce<R>(acc, red);
    if (threadIdx.x < R && r0 + (int)threadIdx.x < n) {
        const size_t at = (size_t)t * n + r0 + threadIdx.x;
        y[at] = add ? add[at] + s : s;
    }
}

// y[t, :] = sum over the slots of weight * out[pair, :], plus the shared expert's rows times sigmoid(logit[t ld]) (logit
// null: as they are) and the rows `add` (may be y).
static __global__ __launch_bounds__(256) void moe_combine_shared(const float *__restrict__ out, const float *__restrict__ wts, int T, int k_used,
                                                                 int h, const float *__restrict__ shared, const float *__restrict__ logit,
                                                                 size_t ld, const float *add, float *y) {
    const size_t total = (size_t)T * h;
    if ((h & 3) == 0) {
        const int per = h / 4;
        const f32x4 *o4 = (const f32x4 *)out, *s4 = (const f32x4 *)shared, *a4 = (const f32x4 *)add;
        for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < total / 4; i += (size_t)gridDim.x * 256) {
            const int t = (int)(i / per), c = (int)(i % per);
            f32x4 acc = add ? a4[i] : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
            for (int s = 0; s < k_used; s++) {
                const f32x4 v = o4[((size_t)t * k_used + s) * per + c];
                const float wt = wts[t * k_used + s];
#pragma unroll
                for (int r = 0; r < 4; r++) acc[r] = fmaf(v[r], wt, acc[r]);
            }
            if (shared) {
                const f32x4 v = s4[i];
                const float wt = logit ? sigmoid_of(logit[t * ld]) : 1.0f;
#pragma unroll
                for (int r = 0; r < 4; r++) acc[r] = fmaf(v[r], wt, acc[r]);
            }
            ((f32x4 *)y)[i] = acc;
        }
        return;
    }
    for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (size_t)gridDim.x * 256) {
        const size_t t = i / h, c = i % h;
        float acc = add ? add[i] : 0.0f;
        for (int s = 0; s < k_used; s++) acc = fmaf(out[(t * k_used + s) * h + c], wts[t * k_used + s], acc);
        if (shared) acc = fmaf(shared[i], logit ? sigmoid_of(logit[t * ld]) : 1.0f, acc);
        y[i] = acc;
    }
}

// ---- GEMM -----------------------------------------------------------------------------------------

struct DenseGemm {
    const uint8_t *A, *W, *W2;     // W2: the up rows of a gated product
    const uint8_t *const *Wp, *const *Wp2;  // grouped: the experts' bases
    uint32_t lda, ldw;             // bytes from a row to the next
    int M, N, stages;              // N: output columns (the gated product reads 2 N weight rows); stages of 128 bytes of k
    int splits;                    // runs of stages, one workgroup each; > 1: C holds the partial sums, [splits][M][width]
    float *C;
    size_t ldc;                    // elements
    // not gated: the results in the element type instead, columns in runs of head_w (a multiple of 4): column c of row r
    // at heads[c / head_w * head_stride + r * head_row + c % head_w]
    void *heads;
    int head_w;
    size_t head_stride, head_row;
    void *act;                     // gated, splits 1: the activations, [M][ld_act] in the element type
    size_t ld_act;
    GatedUnit unit;
    // grouped: rows of A are pairs sorted by expert (group), or their tokens through xsel; results go to yrow of the
    // pair when given, else stay in sorted order
    const int *offsets, *xsel, *yrow;
    int groups, m_tiles;           // m_tiles: row tiles of the grid (grouped: an upper bound)
};

__device__ __forceinline__ void dma_chunk16(const uint8_t *sbase, uint32_t voff, uint32_t lds_base) {
    asm volatile("s_mov_b32 m0, %2\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %0, %1" ::"v"(voff), "s"(sbase),
                 "s"(__builtin_amdgcn_readfirstlane(lds_base))
                 : "memory");
}

// Columns of a partial-sum row: a gated product keeps gate and up in alternating runs of 16.
__host__ __device__ inline size_t gemm_partial_width(int N, bool gated) { return gated ? 2 * (size_t)((N + 15) / 16 * 16) : (size_t)N; }

// BM activation rows x BN weight rows a workgroup of four waves (2 x 2), k in stages of 128 bytes through two LDS
// buffers: the next stage travels global -> LDS (asynchronous 16-byte loads) while the current one is multiplied.
// Chunk c of row r sits at position c ^ (r & 7) of its 128-byte LDS row: the 16 rows a fragment read touches then
// fall into different banks.  The weights are the first operand, so a lane ends with four consecutive columns of
// one activation row.
// GATED: weight rows come in runs of 16 gate rows and the 16 up rows of the same columns.
template <class E, int BM, int BN, bool GATED, bool GROUPED>
__global__ __launch_bounds__(256) void dense_gemm(DenseGemm a) {
    constexpr int STAGE = (BM + BN) * 128, FM = BM / 32, FN = BN / 32;
    __shared__ __attribute__((aligned(128))) uint8_t lds[2 * STAGE];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wm = wave & 1, wn = wave >> 1, g = lane >> 4, l16 = lane & 15;
    // ids 8 apart run on one XCD: give each XCD a contiguous run of tiles (row tiles of one weight tile first), so
    // that a weight tile is read into one L2
    const int n_tiles = (int)gridDim.x / a.m_tiles;  // (gridDim.x = m_tiles * n_tiles)
    const int total = a.m_tiles * n_tiles;
    int id = blockIdx.x;
    if (total >= 16) {
        const int q = total / 8, rem = total % 8, x = id % 8, loc = id / 8;
        id = x * q + min(x, rem) + loc;
    }
    int mt = id % a.m_tiles;
    const int nt = id / a.m_tiles;
    int row_lo = 0, rows_here = a.M;
    const uint8_t *W = a.W, *W2 = a.W2;
    if constexpr (GROUPED) {
        // which expert row tile mt belongs to: lane l counts the tiles of a run of experts
        const int per = (a.groups + 63) / 64;
        int local = 0;
        for (int i = 0; i < per; i++) {
            const int e = lane * per + i;
            if (e < a.groups) local += (a.offsets[e + 1] - a.offsets[e] + BM - 1) / BM;
        }
        int incl = local;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const int v = __shfl_up(incl, off, 64);
            if (lane >= off) incl += v;
        }
        if (mt >= __builtin_amdgcn_readlane(incl, 63)) return;  // past the last tile: the whole workgroup
        int found = -1, first = incl - local;
        if (mt >= first && mt < incl) {
            for (int i = 0; i < per; i++) {
                const int e = lane * per + i, n = e < a.groups ? (a.offsets[e + 1] - a.offsets[e] + BM - 1) / BM : 0;
                if (found < 0 && mt < first + n) found = e;
                else if (found < 0) first += n;
            }
        }
        const int owner = __builtin_ctzll(__ballot(found >= 0));
        const int e = __builtin_amdgcn_readlane(found, owner);
        mt -= __builtin_amdgcn_readlane(first, owner);
        row_lo = a.offsets[e], rows_here = a.offsets[e + 1] - row_lo;
        W = a.Wp[e];
        if constexpr (GATED) W2 = a.Wp2[e];
    }
    const int m0 = mt * BM, c0 = nt * (GATED ? BN / 2 : BN);  // first row within the group, first output column
    const int per_split = (a.stages + a.splits - 1) / a.splits;
    const int st0 = (int)blockIdx.y * per_split, st1 = min(a.stages, st0 + per_split);

    uint32_t va[FM], vw[FN];
#pragma unroll
    for (int i = 0; i < FM; i++) {
        const int row = (tid >> 3) + 32 * i, c = (tid & 7) ^ (row & 7);
        int ar = row_lo + min(m0 + row, rows_here - 1);
        if constexpr (GROUPED) ar = a.xsel ? a.xsel[ar] : ar;
        va[i] = (uint32_t)ar * a.lda + 16u * c;
    }
#pragma unroll
    for (int i = 0; i < FN; i++) {
        const int row = (tid >> 3) + 32 * i, c = (tid & 7) ^ (row & 7);
        const int col = GATED ? c0 + 16 * i + (row & 15) : c0 + row;
        vw[i] = (uint32_t)min(col, a.N - 1) * a.ldw + 16u * c;
    }
    if constexpr (GATED) W = wave < 2 ? W : W2;  // waves 0 and 1 copy rows 0 .. 15 of every 32
    const uint32_t lds0 = (uint32_t)(uintptr_t)lds + (uint32_t)wave * 1024u;
    auto issue = [&](int st, int buf) __attribute__((always_inline)) {
        const uint8_t *pa = a.A + (size_t)st * 128, *pw = W + (size_t)st * 128;
        const uint32_t base = lds0 + (uint32_t)(buf * STAGE);
#pragma unroll
        for (int i = 0; i < FM; i++) dma_chunk16(pa, va[i], base + 4096u * i);
#pragma unroll
        for (int i = 0; i < FN; i++) dma_chunk16(pw, vw[i], base + BM * 128u + 4096u * i);
    };
    f32x4 acc[FN][FM];
#pragma unroll
    for (int n = 0; n < FN; n++)
#pragma unroll
        for (int m = 0; m < FM; m++) acc[n][m] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (st0 < st1) issue(st0, 0);
    for (int st = st0; st < st1; st++) {
        const int buf = (st - st0) & 1;
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();  // everyone's loads of this stage have landed, and the other buffer's readers are done
        if (st + 1 < st1) issue(st + 1, buf ^ 1);
        const uint8_t *la = lds + buf * STAGE + (wm * (BM / 2) + l16) * 128, *lw = lds + buf * STAGE + (BM + wn * (BN / 2) + l16) * 128;
#pragma unroll
        for (int kk = 0; kk < 2; kk++) {
            const int at = 16 * ((4 * kk + g) ^ (l16 & 7));
            u32x4 fa[FM], fw[FN];
#pragma unroll
            for (int m = 0; m < FM; m++) fa[m] = *(const u32x4 *)(la + m * 2048 + at);
#pragma unroll
            for (int n = 0; n < FN; n++) fw[n] = *(const u32x4 *)(lw + n * 2048 + at);
#pragma unroll
            for (int n = 0; n < FN; n++)
#pragma unroll
                for (int m = 0; m < FM; m++) acc[n][m] = E::mma(fw[n], fa[m], acc[n][m]);
        }
    }
    const bool partial = a.splits > 1;
    const size_t width = partial ? gemm_partial_width(a.N, GATED) : a.ldc;
    float *C = a.C + (partial ? (size_t)blockIdx.y * a.M * width : 0);
#pragma unroll
    for (int m = 0; m < FM; m++) {
        const int lr = m0 + wm * (BM / 2) + 16 * m + l16;
        if (lr >= rows_here) continue;
        int orow = row_lo + lr;
        if constexpr (GROUPED) {
            if (a.yrow && !partial) orow = a.yrow[orow];
        }
        if (!GATED && a.heads) {
#pragma unroll
            for (int n = 0; n < FN; n++) {
                const int col = c0 + wn * (BN / 2) + 16 * n + 4 * g;
                if (col >= a.N) continue;  // (N is whole runs)
                typename E::T v[4];
#pragma unroll
                for (int r = 0; r < 4; r++) v[r] = (typename E::T)acc[n][m][r];
                typename E::T *hp = (typename E::T *)a.heads + (size_t)(col / a.head_w) * a.head_stride + (size_t)orow * a.head_row + col % a.head_w;
                __builtin_memcpy(__builtin_assume_aligned(hp, 4 * sizeof(typename E::T)), v, sizeof v);
            }
        } else if (!GATED || partial) {
#pragma unroll
            for (int n = 0; n < FN; n++) {
                const int col = (GATED ? 2 * c0 : c0) + wn * (BN / 2) + 16 * n + 4 * g;
                const int lim = GATED ? (int)width : a.N;
                float *cp = C + (size_t)orow * width + col;
                if (col + 3 < lim && (width & 3) == 0) {
                    *(f32x4 *)cp = acc[n][m];
                } else {
#pragma unroll
                    for (int r = 0; r < 4; r++)
                        if (col + r < lim) cp[r] = acc[n][m][r];
                }
            }
        } else {
#pragma unroll
            for (int q = 0; q < FN / 2; q++) {
                const int col = c0 + wn * (BN / 4) + 16 * q + 4 * g;
                typename E::T v[4];
#pragma unroll
                for (int r = 0; r < 4; r++) v[r] = (typename E::T)a.unit(acc[2 * q][m][r], acc[2 * q + 1][m][r]);
                typename E::T *ap = (typename E::T *)a.act + (size_t)orow * a.ld_act + col;
                if (col + 3 < a.N) {  // (activation rows are whole runs of 64 elements: aligned)
                    __builtin_memcpy(__builtin_assume_aligned(ap, 4 * sizeof(typename E::T)), v, sizeof v);
                } else {
#pragma unroll
                    for (int r = 0; r < 4; r++)
                        if (col + r < a.N) ap[r] = v[r];
                }
            }
        }
    }
}

// The partial sums of a product split over k, in order.
static __global__ __launch_bounds__(256) void gemm_sum_splits(const float *__restrict__ P, int splits, size_t M, int N, float *__restrict__ C,
                                                       size_t ldc) {
    const size_t total = M * (size_t)N;
    for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (size_t)gridDim.x * 256) {
        float s = P[i];
        for (int z = 1; z < splits; z++) s += P[z * total + i];
        C[i / N * ldc + i % N] = s;
    }
}

template <class E>
__global__ __launch_bounds__(256) void gemm_sum_splits_gated(const float *__restrict__ P, int splits, size_t M, int N,
                                                             typename E::T *__restrict__ act, size_t ld_act, GatedUnit unit) {
    const size_t width = gemm_partial_width(N, true), total = M * (size_t)N;
    for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (size_t)gridDim.x * 256) {
        const size_t row = i / N, j = i % N;
        const float *p = P + row * width + 32 * (j / 16) + j % 16;
        float gs = p[0], us = p[16];
        for (int z = 1; z < splits; z++) gs += p[z * M * width], us += p[z * M * width + 16];
        act[row * ld_act + j] = (typename E::T)unit(gs, us);
    }
}

// f32 rows into rows of the element type, padded with zeros.
template <class E>
__global__ __launch_bounds__(256) void rows_to_elem(const float *__restrict__ X, size_t ldx, size_t rows, int k,
                                                    typename E::T *__restrict__ out, size_t stride) {
    const size_t total = rows * stride;
    for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (size_t)gridDim.x * 256) {
        const size_t r = i / stride, c = i % stride;
        out[i] = (typename E::T)(c < (size_t)k ? X[r * ldx + c] : 0.0f);
    }
}

// out[i, :] = W[ids[i], :] * scale in f32 (ids null: row i)
template <class E>
__global__ __launch_bounds__(256) void dense_rows_to_f32(const uint8_t *__restrict__ W, size_t pitch, const uint32_t *__restrict__ ids,
                                                         float *__restrict__ out, size_t rows, int k, float scale) {
    for (size_t r = blockIdx.x; r < rows; r += gridDim.x) {
        const typename E::T *row = (const typename E::T *)(W + (ids ? ids[r] : r) * pitch);
        for (int c = (int)blockIdx.y * 256 + (int)threadIdx.x; c < k; c += (int)gridDim.y * 256) out[r * k + c] = (float)row[c] * scale;
    }
}

// ---- tiles transposed through LDS -----------------------------------------------------------------
//
// 64 rows (tokens) x 64 columns of bf16, a column's tokens side by side: what a product over the tokens reads.  A lane
// brings columns 8 c .. 8 c + 7 of tokens 2 pair and 2 pair + 1 and writes them as eight words.  Column rows are 144 bytes
// apart; runs of 16 bytes are exchanged by the column so that the lanes of a write (8 c's, 8 pairs) meet 64 banks.
constexpr int TILE_COL = 144;  // bytes
__device__ __forceinline__ int tile_word(int c, int e, int pair) { return (8 * c + e) * TILE_COL + 4 * (pair ^ 4 * (c & 6)); }
// tokens 8 j .. 8 j + 7 of a column
__device__ __forceinline__ int tile_chunk(int col, int j) { return col * TILE_COL + 16 * (j ^ (col >> 3 & 6)); }

__device__ __forceinline__ void tile_put(uint8_t *tile, int c, int pair, const u32x4 &a, const u32x4 &b) {
#pragma unroll
    for (int e = 0; e < 8; e++) {
        const uint32_t lo = a[e / 2], hi = b[e / 2];
        *(uint32_t *)(tile + tile_word(c, e, pair)) = e & 1 ? (lo >> 16) | (hi & 0xFFFF0000u) : (lo & 0xFFFFu) | (hi << 16);
    }
}

static __global__ __launch_bounds__(256) void fill_zero(float *__restrict__ p, size_t n) {
    for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) p[i] = 0.0f;
}

}  // namespace jq
