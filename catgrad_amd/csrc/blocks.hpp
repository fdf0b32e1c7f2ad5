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
// Two such products of operands of the same width without norms or biases in one launch; kDeclined: not at once.
int launch_few_rows_linear2(cg_backend *be, const ProductInput (&in)[2], uint32_t rows, const Weight (&w)[2], float *const (&out)[2]);
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
// extra: [rows, slots, width] more terms in words or bfloat16 patterns, added up (null: none); out = x + scale * (all terms)
int launch_gated_sum(cg_backend *be, const Rows &x, const GatedTerm *t, int n, uint32_t rows, uint32_t width, float *out, float scale = 1.0f,
                     const void *extra = nullptr, uint32_t slots = 0, int extra_fmt = kFmtWords);

// ---- embeddings, grouped norms with filters, the tokens' own vectors ---------------------------------------------------
// A table's rows in 32-bit words or bfloat16 patterns.
struct Table {
    const void *p = nullptr;
    int64_t pitch = 0; // elements
    int fmt = kFmtWords;
};
// Token ids in memory, or one id.
struct Tokens {
    const uint32_t *p = nullptr;
    uint32_t value = 0;
};
struct PairEmbeddingPlan {
    uint32_t B, S, width, vocab;
    uint64_t buckets, mul_prev, mul_cur; // multipliers below `buckets`
    Tokens ids, previous;
    uint32_t previous_n;                 // tokens of `previous` per sequence
    Table table, pairs;
    float *out;
    uint32_t *previous_out;
};
int launch_pair_embedding(cg_backend *be, const PairEmbeddingPlan &p);

constexpr uint32_t kMaxTaps = 16;
struct ConvRowsPlan {
    uint32_t B, S, width, groups, taps, run;
    float eps;
    Rows x;
    const float *state; // null: zeros
    float *state_out;   // null with one tap
    int n;
    struct {
        const float *gamma, *conv; // conv null: the norm alone
        void *dst;
        int fmt;    // words or bfloat16 patterns
        bool round; // words: rounded to bfloat16
    } out[2];
};
int launch_conv_rows(cg_backend *be, ConvRowsPlan p);

int launch_side_gate(cg_backend *be, float *g, const Tokens &ids, const Table &table, uint32_t vocab, uint32_t first, uint32_t dim, uint32_t rows);
// A few rows: g[r] = gelu(x[r] . w^T) * the rows' vectors; then out = x + scale * norm(g . w^T) (kDeclined: sizes it does not take).
int launch_side_first(cg_backend *be, const Rows &x, uint32_t rows, const Weight &w, const Tokens &ids, const Table &table, uint32_t vocab, uint32_t first, float *g);
int launch_side_second(cg_backend *be, const Rows &x, const float *g, uint32_t rows, const Weight &w, const float *norm, float eps, float scale, float *out);
int launch_side_sum(cg_backend *be, const Rows &x, const float *y, const float *norm, uint32_t rows, uint32_t width, float eps, float scale, float *out);

// ---- mixtures of experts ---------------------------------------------------------------------------------------------
struct ExpertsPlan {
    uint32_t rows, width, ff, experts, top, groups, keep;
    float limit, slope;
    const void *h;   // [rows, width], words or bfloat16 patterns
    int h_fmt;
    const float *logits, *correction; // correction may be null
    const void *gate_up, *down;       // [experts, 2, ff, width], [experts, width, ff], dense
    int fmt;                          // of the weights
};
// y[r, slot, 0 .. width) = weight * expert of row r's slot-th choice, for any number of rows; words or bfloat16 patterns
int launch_experts(cg_backend *be, const ExpertsPlan &p, float *y, int *y_fmt);
// A few rows: hidden[r, slot, 0 .. ff) (weights applied) and the chosen experts' numbers.
int launch_experts_first(cg_backend *be, const ExpertsPlan &p, float *hidden, uint32_t *chosen);
// out[r] = x[r] + scale * (y[r] . w^T + sum_slot hidden[r, slot] . down[chosen[r, slot]]^T), rows <= kFewRows
int launch_experts_second(cg_backend *be, const ExpertsPlan &p, const float *hidden, const uint32_t *chosen, const Rows &x, const Rows &y, const Weight *w, float scale,
                          float *out);

// ---- attention -------------------------------------------------------------------------------------------------------
struct AttentionPlan {
    uint32_t B, S, heads, kv_heads, dim, vdim;
    uint32_t cached;    // rows of the cache in front of the new ones
    uint32_t window;    // 0: all
    uint64_t position;  // of the first new token
    uint64_t temp_every;
    float temp_coef, scale, eps;
    bool bias, unit_heads, mix_scores, zero_sink;
    uint32_t rot_dims;          // 0: no rotation
    double rot_log2;            // log2 of its base
    const float2 *rot_fine, *rot_coarse; // tables (RotTable); set by launch_attention
    Rows q, k, v;
    const float *q_norm, *k_norm, *talk;
    float *keys, *values;       // row 0 of the cached rows of (b 0, kv head 0); the new rows follow the cached ones
    int64_t k_block, v_block;   // elements from one (b, kv head) to the next
    float *out;                 // [B * S, heads * vdim]
};
#ifdef __HIPCC__
// {cos, sin} of pair i at a position
__device__ __forceinline__ float2 rotation_at(const AttentionPlan &p, uint64_t position, uint32_t i) {
    const uint32_t pairs = p.rot_dims / 2;
    const float2 a = p.rot_fine[(position % kRotFine) * pairs + i], b = p.rot_coarse[(position / kRotFine) * pairs + i];
    return make_float2(fmaf(a.x, b.x, -a.y * b.y), fmaf(a.x, b.y, a.y * b.x));
}
#endif
int launch_attention(cg_backend *be, const AttentionPlan &p);
// More than a few new tokens, on the matrix instructions (q: the prepared queries); kDeclined: sizes it does not take.
int launch_attention_tiles(cg_backend *be, const AttentionPlan &p, const float *q);
// Soft-max over mixed scores (block_attention_mixed.hip).  `scores`: the scores' segments as attention_scores_kernel leaves
// them, of the rows row0 .. row0 + rows - 1; parts / part_stats: memory of nseg results per (row, head).
int launch_mixed_rows(cg_backend *be, const AttentionPlan &p, uint32_t row0, uint32_t rows, uint32_t nseg, const float *scores, float *parts, float2 *part_stats);
int launch_mixed_tiles(cg_backend *be, const AttentionPlan &p, const float *q);
int launch_mixed_step(cg_backend *be, const AttentionPlan &p);

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
