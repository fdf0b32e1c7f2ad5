// Launchers of the decoder blocks' kernels (the last section of include/catgrad_hip.h), called by blocks.cpp.
#pragma once

#include "common.hpp"

namespace cg {

// Activations [B, S, features] as rows: row r = b * S + s begins at p + r * pitch.
struct Rows {
    const float *p = nullptr;
    int64_t pitch = 0;
};

// A weight matrix [N, K] with its rows dense or pitched, in 32-bit words or bfloat16 patterns.
struct Weight {
    const void *p = nullptr;
    int64_t pitch = 0; // elements
    int fmt = kFmtWords;
    uint32_t n = 0, k = 0;
};

// The left operand of a product as its kernels load it: (x | x2) with the RMS norm (gamma) or the polynomial norm (poly)
// applied, neither, but not both.
struct ProductInput {
    Rows x, x2;
    uint32_t k1 = 0, k = 0; // columns of x, of both
    const float *gamma = nullptr, *poly = nullptr;
    float eps = 0.0f;
};

constexpr uint32_t kFewRows = 8;           // rows that a product takes on the weight-streaming kernels
constexpr uint32_t kFewRowsLds = 96 << 10; // bytes of LDS that their operands may take
// The compiled row count that takes `rows` rows of `bytes_per_row` bytes of LDS each; 0: none does.
inline uint32_t few_rows_slots(uint64_t rows, uint64_t bytes_per_row) {
    for (uint32_t m : {1u, 2u, 4u, 8u})
        if (m >= rows && m * bytes_per_row <= kFewRowsLds) return m;
    return 0;
}
inline uint32_t staged_pitch(uint32_t k) { return (k + 7) / 8 * 8; } // floats of a staged row

// out[r, n] = scale * in[r, :] . w[n, :] + bias[n], rows <= kFewRows
int launch_few_rows_linear(cg_backend *be, const ProductInput &in, uint32_t rows, const Weight &w, const float *bias, float scale, float *out);
// out[r, n] = x[r, n] + sum_i sigmoid(gate_i[r, n] + gate_bias_i[n]) * (in_i[r, :] . w_i[n, :]), rows <= kFewRows
struct ResidualBranch {
    ProductInput in;
    Weight w;
    Rows gate; // p null: none
    const float *gate_bias = nullptr;
};
// Whether launch_few_rows_residual takes these branches (one of them with 16-byte rows at most four rows deep, or LDS for all)
bool takes_few_rows_residual(const ResidualBranch *br, int n, uint32_t rows);
int launch_few_rows_residual(cg_backend *be, const Rows &x, const ResidualBranch *br, int n, uint32_t rows, uint32_t width, float *out);

// y[rows, w.n] = x . w^T of dense bfloat16 patterns x [rows, w.k] on 128-wide tiles; kDeclined: operands it does not take.
int launch_bf16_tiles(cg_backend *be, const void *x, uint32_t rows, const Weight &w, float *y);
bool takes_bf16_tiles(uint32_t rows, const Weight &w);

// dst[r, 0 .. k) = the product input of row r, as 32-bit words (bf16: rounded to it first) or bfloat16 patterns
int launch_product_input(cg_backend *be, const ProductInput &in, uint32_t rows, void *dst, bool round_bf16, int fmt);
// y[r, n] = y[r, n] * scale + bias[n] in place
int launch_affine_rows(cg_backend *be, float *y, uint32_t rows, uint32_t n, const float *bias, float scale);
// out = x + sum_i sigmoid(gate_i + bias_i) * y_i
struct GatedTerm {
    const float *y = nullptr;
    Rows gate;
    const float *gate_bias = nullptr;
};
int launch_gated_sum(cg_backend *be, const Rows &x, const GatedTerm *t, int n, uint32_t rows, uint32_t width, float *out);

// ---- attention -------------------------------------------------------------------------------------------------------
struct AttentionPlan {
    uint32_t B, S, heads, kv_heads, dim, vdim;
    uint32_t cached;    // rows of the cache in front of the new ones
    uint32_t window;    // 0: all
    uint64_t position;  // of the first new token
    uint64_t temp_every;
    float temp_coef, scale, eps;
    bool bias;
    Rows q, k, v;
    const float *q_norm, *k_norm, *talk;
    float *keys, *values;       // row 0 of the cached rows of (b 0, kv head 0); the new rows follow the cached ones
    int64_t k_block, v_block;   // elements from one (b, kv head) to the next
    float *out;                 // [B * S, heads * vdim]
};
int launch_attention(cg_backend *be, const AttentionPlan &p);
// More than a few new tokens, on the matrix instructions (q: the prepared queries); kDeclined: sizes it does not take.
int launch_attention_tiles(cg_backend *be, const AttentionPlan &p, const float *q);

// ---- gated delta rule ------------------------------------------------------------------------------------------------
struct DeltaPlan {
    uint32_t B, S, heads, kv_heads, dim, vdim, taps;
    float eps;
    Rows q, k, v, beta, decay, gate; // decay, gate: what goes through decay_w / gate_w
    uint32_t decay_rank, gate_rank;
    const float *conv_q, *conv_k, *conv_v, *decay_w, *gate_w, *a_log, *dt_bias, *norm;
    const float *state, *conv_state; // null: zeros
    float *out, *state_out, *conv_out;
};
int launch_channel_delta(cg_backend *be, const DeltaPlan &p);

} // namespace cg
