// Launches of the products with plain weight rows (kernels_dense.hpp) and of the residual update in front of them.
#pragma once
#include "kernels_dense.hpp"
#include "moe.hpp"

namespace jqh {

constexpr int GEMV_MAX_ROWS = 8;   // activation rows up to which a product runs on the GEMV, in f32 activations
constexpr int NORM_MAX_WIDTH = 16384;
constexpr int FUSED_NORM_MAX_WIDTH = 8192;

// Y[t, :] = X[t, :] W^T for T <= GEMV_MAX_ROWS.  With `nm` (one row, width = W's k, at most FUSED_NORM_MAX_WIDTH) X
// is the row nm makes; nm->x_out must not be nm->x then.
int dense_gemv(const jq_weight *w, const float *X, size_t ldx, int T, float *Y, size_t ldy, hipStream_t s,
               const jq::ResidualNorm *nm = nullptr);
int dense_gemv_gated(const jq_weight *gate, const jq_weight *up, const float *X, size_t ldx, int T, float *Y, size_t ldy,
                     const jq::GatedUnit &unit, hipStream_t s, const jq::ResidualNorm *nm = nullptr);
// The same for any T over activations in the weights' type, rows `lda` elements apart (whole runs of 64, numbers behind
// the k-th up to the next whole run); the gated product leaves its activations in that form too.
int dense_gemm(const jq_weight *w, const void *A, size_t lda, int T, float *C, size_t ldc, hipStream_t s);
// The same with the results in the weights' type, by heads of `head_w` columns (a multiple of 4; n is whole heads): column c
// of row t at out[c / head_w * head_stride + t * head_row + c % head_w], strides in elements, multiples of 4.  w_row: the first
// of the `n` rows of w to take.
int dense_gemm_heads(const jq_weight *w, size_t w_row, size_t n, const void *A, size_t lda, int T, void *out, int head_w, size_t head_stride,
                     size_t head_row, hipStream_t s);
int dense_gemm_gated(const jq_weight *gate, const jq_weight *up, const void *A, size_t lda, int T, void *act, size_t ld_act,
                     const jq::GatedUnit &unit, hipStream_t s);
// f32 rows in and out, rows packed: what jq_matmul_t runs for these types.
int dense_matmul(uint32_t type, const uint8_t *W, size_t row_bytes, const float *X, float *Y, size_t m, size_t k, size_t n,
                 hipStream_t s);
// Rows of W (those ids name, or the first `rows`) times scale, in f32.
int dense_decode(const jq_weight *w, const uint32_t *ids, float *out, size_t rows, float scale, hipStream_t s);
// The residual update over `rows` rows; `type` is the element type of `he` (see residual_norm_rows).
int residual_norm(const jq::ResidualNorm &a, uint32_t type, void *he, size_t stride, size_t rows, const uint32_t *at, hipStream_t s);
int zero_floats(float *p, size_t n, hipStream_t s);
int rows_to_elem(uint32_t type, const float *X, size_t ldx, size_t rows, int k, void *out, size_t stride, hipStream_t s);

// The layer with BF16 / F32 experts over x [T, hidden] in f32 and, when the caller has them, the same rows in the
// experts' type (xe, rows dense_stride(hidden) apart; x may then be null for calls that are not decode-sized).
struct MoeDenseExtras {
    const jq::ResidualNorm *pre = nullptr;  // one token: the router launch makes x (pre->h_out == x)
    // logits made elsewhere, `ld` floats from a token to the next: the router's, and the shared expert's gate
    const float *logits = nullptr, *shared_logit = nullptr;
    size_t ld = 0;
    const float *add = nullptr;             // rows that join the result (may be y)
    // one token, decode-sized: another product W mid that joins the result
    const jq_weight *W = nullptr;
    const float *mid = nullptr;
};
int moe_forward_dense(jq_moe *m, size_t T, const float *x, const void *xe, float *y, hipStream_t s, const MoeDenseExtras &ex = MoeDenseExtras());
// Whether T tokens run on the decode-sized kernels.
bool moe_dense_decode_sized(const jq_moe *m, size_t T);
bool moe_dense_fuses_norm(const jq_moe *m, size_t T);

}  // namespace jqh
