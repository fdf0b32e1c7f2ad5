// Row-wise kernels of the decoder blocks: products of a few rows with streamed weight matrices (the norms of their left
// operand in the loads, the gated residual sum in the store), and for many rows the operand and the sum on their own.
#include "blocks.hpp"
#include "device_utils.hpp"

#include <algorithm>

namespace cg {
namespace {

constexpr int kThreads = 256, kWaves = 4;

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int d = 32; d > 0; d >>= 1) v += __shfl_xor(v, d, 64);
    return v;
}
// sum over the 256 threads of a workgroup, for every thread; `red` has a slot per wave
__device__ __forceinline__ float block_sum(float v, float *red) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}
__device__ __forceinline__ float sigmoid(float z) { // on the hardware's exp2 and reciprocal
    return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(z * -1.44269504088896341f));
}
__device__ __forceinline__ float bf16_lo(uint32_t w) { return asf(w << 16); }
__device__ __forceinline__ float bf16_hi(uint32_t w) { return asf(w & 0xFFFF0000u); }

__device__ __forceinline__ float input_at(const ProductInput &in, uint32_t r, uint32_t k) {
    return k < in.k1 ? in.x.p[(int64_t)r * in.x.pitch + k] : in.x2.p[(int64_t)r * in.x2.pitch + (k - in.k1)];
}

// What a row of the input is multiplied by / turned into, from sums over the row.
struct RowScale {
    float s1 = 1.0f, s2 = 0.0f, s3 = 0.0f, c = 0.0f; // gamma: s1 = 1 / rms; poly: z -> s1 z + s2 z^2 + s3 z^3 + c
};
__device__ __forceinline__ RowScale row_scale(const ProductInput &in, float m1, float m2, float m3) {
    RowScale o;
    const float n = (float)in.k;
    if (in.gamma) {
        o.s1 = 1.0f / sqrtf(m1 / n + in.eps);
    } else if (in.poly) {
        o.s1 = in.poly[0] / sqrtf(m1 / n + in.eps);
        o.s2 = in.poly[1] / sqrtf(m2 / n + in.eps);
        o.s3 = in.poly[2] / sqrtf(m3 / n + in.eps);
        o.c = in.poly[3];
    }
    return o;
}
__device__ __forceinline__ float scaled(const ProductInput &in, const RowScale &o, float z, uint32_t k) {
    if (in.gamma) return z * o.s1 * in.gamma[k];
    if (in.poly) return fmaf(z, fmaf(z, fmaf(z, o.s3, o.s2), o.s1), o.c);
    return z;
}

// Where column k of a staged row lies in LDS: for bfloat16 weights, which a lane takes eight columns at a time, the two
// halves of every eight apart, so that both 16-byte reads of a wave are contiguous.
template <bool BF16> __device__ __forceinline__ uint32_t lds_at(uint32_t k, uint32_t half) {
    return BF16 ? ((k >> 2) & 1) * half + ((k >> 3) << 2) + (k & 3) : k;
}

// The rows of the product's left operand into LDS, [M][pitch]; columns up to the pitch are zero.
template <int M, bool BF16> __device__ void stage_input(const ProductInput &in, uint32_t rows, uint32_t pitch, float *lds, float *red) {
    const uint32_t half = pitch / 2;
    float m1[M], m2[M], m3[M];
#pragma unroll
    for (int m = 0; m < M; m++) m1[m] = m2[m] = m3[m] = 0.0f;
    for (uint32_t k = threadIdx.x; k < pitch; k += kThreads) {
        const uint32_t at = lds_at<BF16>(k, half);
#pragma unroll
        for (int m = 0; m < M; m++) {
            const float z = k < in.k && m < (int)rows ? input_at(in, m, k) : 0.0f;
            lds[m * pitch + at] = z;
            const float z2 = z * z;
            m1[m] += z2;
            if (in.poly) {
                m2[m] = fmaf(z2, z2, m2[m]);
                m3[m] = fmaf(z2 * z2, z2, m3[m]);
            }
        }
    }
    if (!in.gamma && !in.poly) return; // (the caller's barrier follows)
    RowScale o[M];
#pragma unroll
    for (int m = 0; m < M; m++) {
        const float a = block_sum(m1[m], red), b = in.poly ? block_sum(m2[m], red) : 0.0f, c = in.poly ? block_sum(m3[m], red) : 0.0f;
        o[m] = row_scale(in, a, b, c);
    }
    for (uint32_t k = threadIdx.x; k < in.k; k += kThreads) { // every thread its own columns again
        const uint32_t at = lds_at<BF16>(k, half);
#pragma unroll
        for (int m = 0; m < M; m++) lds[m * pitch + at] = scaled(in, o[m], lds[m * pitch + at], k);
    }
}

// What a lane holds of NC weight rows: 16 bytes of each, or one element.
template <int NC, bool BF16, bool VEC> struct WeightRegs {
    uint4 v[NC];
    __device__ __forceinline__ void load(const Weight &w, const uint32_t (&n)[NC], uint32_t k) {
        if constexpr (VEC) {
            constexpr uint32_t EB = BF16 ? 2 : 4;
#pragma unroll
            for (int c = 0; c < NC; c++) {
                typedef uint32_t u4 __attribute__((ext_vector_type(4)));
                const u4 t = __builtin_nontemporal_load(reinterpret_cast<const u4 *>(static_cast<const char *>(w.p) + ((int64_t)n[c] * w.pitch + k) * EB));
                v[c] = make_uint4(t[0], t[1], t[2], t[3]);
            }
        } else {
#pragma unroll
            for (int c = 0; c < NC; c++)
                v[c].x = BF16 ? (uint32_t)static_cast<const uint16_t *>(w.p)[(int64_t)n[c] * w.pitch + k] << 16
                              : static_cast<const uint32_t *>(w.p)[(int64_t)n[c] * w.pitch + k];
        }
    }
};

// acc[c][m] += w[n_c, :] . lds[m, :]; a wave walks all of K.  `first` holds the first trip's weights already.
template <int M, int NC, bool BF16, bool VEC>
__device__ __forceinline__ void dot_rows(const Weight &w, const uint32_t (&n)[NC], const float *lds, uint32_t pitch, WeightRegs<NC, BF16, VEC> cur,
                                         float (&acc)[NC][M]) {
    constexpr uint32_t VW = VEC ? (BF16 ? 8 : 4) : 1, STEP = 64 * VW;
    const uint32_t half = pitch / 2;
    uint32_t k = (threadIdx.x & 63) * VW;
    while (k < w.k) {
        WeightRegs<NC, BF16, VEC> next;
        if (k + STEP < w.k) next.load(w, n, k + STEP);
        if constexpr (!VEC) {
#pragma unroll
            for (int m = 0; m < M; m++) {
                const float x = lds[m * pitch + lds_at<BF16>(k, half)];
#pragma unroll
                for (int c = 0; c < NC; c++) acc[c][m] = fmaf(asf(cur.v[c].x), x, acc[c][m]);
            }
        } else if constexpr (BF16) {
#pragma unroll
            for (int m = 0; m < M; m++) {
                const float4 a = *reinterpret_cast<const float4 *>(lds + m * pitch + (k >> 1)), b = *reinterpret_cast<const float4 *>(lds + m * pitch + half + (k >> 1));
#pragma unroll
                for (int c = 0; c < NC; c++) {
                    float s = acc[c][m];
                    s = fmaf(bf16_lo(cur.v[c].x), a.x, s);
                    s = fmaf(bf16_hi(cur.v[c].x), a.y, s);
                    s = fmaf(bf16_lo(cur.v[c].y), a.z, s);
                    s = fmaf(bf16_hi(cur.v[c].y), a.w, s);
                    s = fmaf(bf16_lo(cur.v[c].z), b.x, s);
                    s = fmaf(bf16_hi(cur.v[c].z), b.y, s);
                    s = fmaf(bf16_lo(cur.v[c].w), b.z, s);
                    s = fmaf(bf16_hi(cur.v[c].w), b.w, s);
                    acc[c][m] = s;
                }
            }
        } else {
#pragma unroll
            for (int m = 0; m < M; m++) {
                const float4 a = *reinterpret_cast<const float4 *>(lds + m * pitch + k);
#pragma unroll
                for (int c = 0; c < NC; c++) {
                    float s = acc[c][m];
                    s = fmaf(asf(cur.v[c].x), a.x, s);
                    s = fmaf(asf(cur.v[c].y), a.y, s);
                    s = fmaf(asf(cur.v[c].z), a.z, s);
                    s = fmaf(asf(cur.v[c].w), a.w, s);
                    acc[c][m] = s;
                }
            }
        }
        cur = next;
        k += STEP;
    }
}

template <int NC> __device__ __forceinline__ void wave_columns(uint32_t N, uint32_t (&n)[NC], uint32_t *n0) {
    *n0 = (blockIdx.x * kWaves + (threadIdx.x >> 6)) * NC;
#pragma unroll
    for (int c = 0; c < NC; c++) n[c] = min(*n0 + c, N - 1);
}

template <int M, int NC, bool BF16, bool VEC>
__global__ __launch_bounds__(kThreads) void few_rows_linear_kernel(const ProductInput in, const uint32_t rows, const Weight w, const uint32_t pitch,
                                                                   const float *__restrict__ bias, const float scale, float *__restrict__ out) {
    extern __shared__ float lds[];
    __shared__ float red[kWaves];
    uint32_t n[NC], n0;
    wave_columns<NC>(w.n, n, &n0);
    constexpr uint32_t VW = VEC ? (BF16 ? 8 : 4) : 1;
    WeightRegs<NC, BF16, VEC> first;
    if ((threadIdx.x & 63) * VW < w.k) first.load(w, n, (threadIdx.x & 63) * VW); // on its way while the operand is staged
    stage_input<M, BF16>(in, rows, pitch, lds, red);
    __syncthreads();
    float acc[NC][M] = {};
    dot_rows<M, NC, BF16, VEC>(w, n, lds, pitch, first, acc);
#pragma unroll
    for (int c = 0; c < NC; c++) {
#pragma unroll
        for (int m = 0; m < M; m++) {
            const float s = wave_sum(acc[c][m]);
            if ((threadIdx.x & 63) == (uint32_t)m && m < (int)rows && n0 + c < w.n)
                out[(int64_t)m * w.n + n0 + c] = s * scale + (bias ? bias[n0 + c] : 0.0f);
        }
    }
}

template <int M, bool BF16, bool VEC, int NB>
__global__ __launch_bounds__(kThreads) void few_rows_residual_kernel(const Rows x, const ResidualBranch b0, const ResidualBranch b1, const uint32_t rows,
                                                                     const uint32_t width, const uint32_t pitch0, const uint32_t pitch1,
                                                                     float *__restrict__ out) {
    extern __shared__ float lds[];
    __shared__ float red[kWaves];
    uint32_t n[1], n0;
    wave_columns<1>(width, n, &n0);
    constexpr uint32_t VW = VEC ? (BF16 ? 8 : 4) : 1;
    const uint32_t k0 = (threadIdx.x & 63) * VW;
    WeightRegs<1, BF16, VEC> f0, f1;
    if (k0 < b0.w.k) f0.load(b0.w, n, k0);
    if (NB > 1 && k0 < b1.w.k) f1.load(b1.w, n, k0);
    float *lds1 = lds + M * pitch0;
    stage_input<M, BF16>(b0.in, rows, pitch0, lds, red);
    if (NB > 1) stage_input<M, BF16>(b1.in, rows, pitch1, lds1, red);
    // the lane that stores row m asks for the rest of the sum now
    const uint32_t lane = threadIdx.x & 63, m_of = min(lane, rows - 1);
    const float xs = x.p[(int64_t)m_of * x.pitch + n[0]];
    const float g0 = b0.gate.p ? b0.gate.p[(int64_t)m_of * b0.gate.pitch + n[0]] + (b0.gate_bias ? b0.gate_bias[n[0]] : 0.0f) : 0.0f;
    const float g1 = NB > 1 && b1.gate.p ? b1.gate.p[(int64_t)m_of * b1.gate.pitch + n[0]] + (b1.gate_bias ? b1.gate_bias[n[0]] : 0.0f) : 0.0f;
    __syncthreads();
    float a0[1][M] = {}, a1[1][M] = {};
    dot_rows<M, 1, BF16, VEC>(b0.w, n, lds, pitch0, f0, a0);
    if (NB > 1) dot_rows<M, 1, BF16, VEC>(b1.w, n, lds1, pitch1, f1, a1);
    float s0 = 0.0f, s1 = 0.0f;
#pragma unroll
    for (int m = 0; m < M; m++) {
        const float t0 = wave_sum(a0[0][m]), t1 = NB > 1 ? wave_sum(a1[0][m]) : 0.0f;
        if (lane == (uint32_t)m) {
            s0 = t0;
            s1 = t1;
        }
    }
    if (lane < rows && n0 < width) {
        float o = b0.gate.p ? sigmoid(g0) * s0 : s0;
        if (NB > 1) o += b1.gate.p ? sigmoid(g1) * s1 : s1;
        out[(int64_t)lane * width + n0] = xs + o;
    }
}

// ---- at most four rows -----------------------------------------------------------------------------------------------
// The 4x4x4 (bfloat16) and 4x4x1 (f32) matrix instructions multiply 16 independent blocks of four columns and four rows:
// lane (block = lane / 4, j = lane % 4) supplies weights of column n0 + j and activations of row j at the block's values of
// k, 16 bytes of weights at a time, and finds rows 0 .. 3 ... of its column j's sums in its registers — the sums over the
// blocks, and over the waves of the workgroup, which take k in turn, come at the end.  Nothing is staged and nothing waits:
// the factors of a norm are the same for a whole row, so they are applied to the sums, and the row sums they need are formed
// from what a wave loads anyway.  The polynomial norm is linear in z, z^2, z^3 and 1: four sums instead of one.
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef short bf16x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bfx2 __attribute__((ext_vector_type(2)));

template <bool BF16> struct Frag { // a lane's weights, or its activations in the form the instruction takes
    static constexpr uint32_t W = BF16 ? 8 : 4; // values of k
    uint32_t v[4];
};

template <bool BF16> __device__ __forceinline__ Frag<BF16> load_weights(const Weight &w, uint32_t n, uint32_t k) {
    typedef uint32_t u4 __attribute__((ext_vector_type(4)));
    Frag<BF16> f;
    k = min(k, w.k - Frag<BF16>::W); // (behind the last column the activations are zero: no load waits for a test)
    const u4 t = __builtin_nontemporal_load(reinterpret_cast<const u4 *>(static_cast<const char *>(w.p) + ((int64_t)n * w.pitch + k) * (BF16 ? 2 : 4)));
#pragma unroll
    for (int i = 0; i < 4; i++) f.v[i] = t[i];
    return f;
}
template <bool BF16> __device__ __forceinline__ Frag<BF16> pack(const float (&x)[Frag<BF16>::W]) {
    Frag<BF16> f;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        if constexpr (BF16) {
            typedef float f2 __attribute__((ext_vector_type(2)));
            const f2 t = {x[2 * i], x[2 * i + 1]};
            f.v[i] = __builtin_bit_cast(uint32_t, __builtin_convertvector(t, bfx2));
        } else {
            f.v[i] = asu(x[i]);
        }
    }
    return f;
}
template <bool BF16> __device__ __forceinline__ f32x4 multiply(const Frag<BF16> &w, const Frag<BF16> &x, f32x4 acc) {
    if constexpr (BF16) {
#pragma unroll
        for (int i = 0; i < 4; i += 2) {
            typedef uint32_t u2 __attribute__((ext_vector_type(2)));
            const u2 a = {w.v[i], w.v[i + 1]}, b = {x.v[i], x.v[i + 1]};
            acc = __builtin_amdgcn_mfma_f32_4x4x4bf16_1k(__builtin_bit_cast(bf16x4, a), __builtin_bit_cast(bf16x4, b), acc, 0, 0, 0);
        }
    } else {
#pragma unroll
        for (int i = 0; i < 4; i++) acc = __builtin_amdgcn_mfma_f32_4x4x1f32(asf(w.v[i]), asf(x.v[i]), acc, 0, 0, 0);
    }
    return acc;
}
// W consecutive activations of row r (zeros behind the last column and for rows that are not there)
template <bool BF16> __device__ __forceinline__ void load_input(const ProductInput &in, uint32_t r, bool there, uint32_t k, float (&x)[Frag<BF16>::W]) {
#pragma unroll
    for (uint32_t i = 0; i < Frag<BF16>::W; i += 4) {
        const uint32_t at = min(k + i, in.k - 4);
        const float *first = in.x.p + (int64_t)r * in.x.pitch + at, *second = in.x2.p + (int64_t)r * in.x2.pitch + at - in.k1;
        const f32x4 t = *reinterpret_cast<const f32x4 *>(at < in.k1 ? first : second);
        const bool in_row = there && k + i < in.k;
#pragma unroll
        for (int j = 0; j < 4; j++) x[i + j] = in_row ? t[j] : 0.0f;
    }
}
// over the 16 lanes that share j
__device__ __forceinline__ float blocks_sum(float v) {
#pragma unroll
    for (int d = 4; d < 64; d <<= 1) v += __shfl_xor(v, d, 64);
    return v;
}

// A workgroup holds all of its waves' activations in registers (STEPS of 64 lanes' worth each) and walks column groups.
template <bool BF16, int STEPS, int WAVES>
__device__ __forceinline__ void four_rows_linear(const ProductInput &in, const uint32_t rows, const Weight &w, const uint32_t block, const uint32_t iters,
                                                 const float *__restrict__ bias, const float scale, float *__restrict__ out) {
    constexpr uint32_t W = Frag<BF16>::W, SPAN = 16 * W;
    __shared__ f32x4 sums[2][WAVES][4];
    __shared__ float squares[WAVES][4];
    const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63, j = lane & 3, k0 = wave * SPAN + (lane >> 2) * W;
    const uint32_t g0 = block * iters, groups = (w.n + 3) / 4, g1 = min(g0 + iters, groups);
    Frag<BF16> wt[STEPS];
    auto ask = [&](uint32_t g) {
        const uint32_t n = min(g * 4 + j, w.n - 1);
#pragma unroll
        for (int s = 0; s < STEPS; s++) wt[s] = load_weights<BF16>(w, n, k0 + s * WAVES * SPAN);
    };
    ask(g0);
    Frag<BF16> x[STEPS];
    float ss = 0.0f;
#pragma unroll
    for (int s = 0; s < STEPS; s++) {
        const uint32_t k = k0 + s * WAVES * SPAN;
        float z[W];
        load_input<BF16>(in, min(j, rows - 1), j < rows, k, z);
        if (in.gamma) {
#pragma unroll
            for (uint32_t i = 0; i < W; i++) {
                ss = fmaf(z[i], z[i], ss);
                z[i] *= in.gamma[min(k + i, in.k - 1)];
            }
        }
        x[s] = pack<BF16>(z);
    }
    if (in.gamma) {
        ss = blocks_sum(ss);
        if (lane < 4) squares[wave][lane] = ss;
    }
    float rstd = scale;
    for (uint32_t g = g0; g < g1; g++) {
        f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int s = 0; s < STEPS; s++) acc = multiply<BF16>(wt[s], x[s], acc);
        if (g + 1 < g1) ask(g + 1);
#pragma unroll
        for (int r = 0; r < 4; r++) acc[r] = blocks_sum(acc[r]);
        f32x4(&mine)[WAVES][4] = sums[g & 1];
        if (lane < 4) mine[wave][lane] = acc;
        __syncthreads(); // (two buffers: the next group's sums do not wait for these to be read)
        if (wave == (g - g0) % WAVES && lane < 16) { // lane (j, r): row j, column r of the group
            const uint32_t m = lane >> 2, c = lane & 3, n = g * 4 + c;
            float s = 0.0f;
#pragma unroll
            for (int i = 0; i < WAVES; i++) s += mine[i][m][c];
            if (in.gamma) {
                float q = 0.0f;
#pragma unroll
                for (int i = 0; i < WAVES; i++) q += squares[i][m];
                rstd = scale / sqrtf(q / (float)in.k + in.eps);
            }
            if (m < rows && n < w.n) out[(int64_t)m * w.n + n] = s * rstd + (bias ? bias[n] : 0.0f);
        }
    }
}

template <bool BF16, int STEPS, int WAVES>
__global__ __launch_bounds__(WAVES * 64) void four_rows_linear_kernel(const ProductInput in, const uint32_t rows, const Weight w, const uint32_t iters,
                                                                      const float *__restrict__ bias, const float scale, float *__restrict__ out) {
    four_rows_linear<BF16, STEPS, WAVES>(in, rows, w, blockIdx.x, iters, bias, scale, out);
}
// two products, the first on the first blocks0 workgroups
struct FourRowsJob {
    ProductInput in;
    Weight w;
    float *out;
    uint32_t iters;
};
template <bool BF16, int STEPS, int WAVES>
__global__ __launch_bounds__(WAVES * 64) void four_rows_linear2_kernel(const FourRowsJob j0, const FourRowsJob j1, const uint32_t blocks0, const uint32_t rows) {
    if (blockIdx.x < blocks0) four_rows_linear<BF16, STEPS, WAVES>(j0.in, rows, j0.w, blockIdx.x, j0.iters, nullptr, 1.0f, j0.out);
    else four_rows_linear<BF16, STEPS, WAVES>(j1.in, rows, j1.w, blockIdx.x - blocks0, j1.iters, nullptr, 1.0f, j1.out);
}

// One branch of the residual sum: the sums of the polynomial's terms (or the plain sum) and the row sums they are scaled by.
template <int NG> struct BranchSums {
    f32x4 acc[NG][4]; // of z, z^2, z^3, 1
    float m[3];
};
template <bool BF16, int NG, int WAVES, bool POLY>
__device__ __forceinline__ void walk_branch(const ResidualBranch &b, uint32_t rows, uint32_t width, uint32_t n0, BranchSums<NG> &o) {
    constexpr uint32_t W = Frag<BF16>::W, SPAN = 16 * W, STEP = WAVES * SPAN;
    constexpr int AHEAD = 4;
    const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63, j = lane & 3;
    uint32_t n[NG];
#pragma unroll
    for (int g = 0; g < NG; g++) n[g] = min(n0 + 4 * g + j, width - 1);
    float one[W];
#pragma unroll
    for (uint32_t i = 0; i < W; i++) one[i] = 1.0f;
    const Frag<BF16> ones = pack<BF16>(one);
    for (uint32_t base = wave * SPAN; base < b.w.k; base += AHEAD * STEP) { // (the same trips for every lane: the instruction does not mask)
        const uint32_t k0 = base + (lane >> 2) * W;
        Frag<BF16> wt[AHEAD][NG];
        float z[AHEAD][W];
#pragma unroll
        for (int a = 0; a < AHEAD; a++)
#pragma unroll
            for (int g = 0; g < NG; g++) wt[a][g] = load_weights<BF16>(b.w, n[g], k0 + a * STEP);
#pragma unroll
        for (int a = 0; a < AHEAD; a++) load_input<BF16>(b.in, min(j, rows - 1), j < rows, k0 + a * STEP, z[a]);
#pragma unroll
        for (int a = 0; a < AHEAD; a++) {
            Frag<BF16> x = pack<BF16>(z[a]);
#pragma unroll
            for (int g = 0; g < NG; g++) o.acc[g][0] = multiply<BF16>(wt[a][g], x, o.acc[g][0]);
            if constexpr (POLY) {
                float p[W], c[W];
#pragma unroll
                for (uint32_t i = 0; i < W; i++) {
                    p[i] = z[a][i] * z[a][i];
                    c[i] = p[i] * z[a][i];
                    o.m[0] += p[i];
                    o.m[1] = fmaf(p[i], p[i], o.m[1]);
                    o.m[2] = fmaf(c[i], c[i], o.m[2]);
                }
                x = pack<BF16>(p);
#pragma unroll
                for (int g = 0; g < NG; g++) o.acc[g][1] = multiply<BF16>(wt[a][g], x, o.acc[g][1]);
                x = pack<BF16>(c);
#pragma unroll
                for (int g = 0; g < NG; g++) o.acc[g][2] = multiply<BF16>(wt[a][g], x, o.acc[g][2]);
#pragma unroll
                for (int i = 0; i < 4; i++) x.v[i] = k0 + a * STEP < b.w.k ? ones.v[i] : 0;
#pragma unroll
                for (int g = 0; g < NG; g++) o.acc[g][3] = multiply<BF16>(wt[a][g], x, o.acc[g][3]);
            }
        }
    }
}

// NG groups of four columns per workgroup.  POLY: branch 1 (or the only one) goes through the polynomial norm.
template <bool BF16, int NB, int NG, int WAVES, bool POLY0, bool POLY1>
__global__ __launch_bounds__(WAVES * 64) void four_rows_residual_kernel(const Rows x, const ResidualBranch b0, const ResidualBranch b1, const uint32_t rows,
                                                                        const uint32_t width, float *__restrict__ out) {
    __shared__ f32x4 sums[NB][WAVES][NG][4][4]; // [branch][wave][group][term][row]
    __shared__ float squares[NB][WAVES][3][4];
    const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63, n0 = blockIdx.x * NG * 4;
    BranchSums<NG> s[NB];
#pragma unroll
    for (int b = 0; b < NB; b++) {
#pragma unroll
        for (int t = 0; t < 4; t++)
#pragma unroll
            for (int g = 0; g < NG; g++) s[b].acc[g][t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
        s[b].m[0] = s[b].m[1] = s[b].m[2] = 0.0f;
    }
    // thread e of the first 16 * NG: row m, column n; what it needs besides the sums is asked for first
    const uint32_t e = threadIdx.x, m = e / (4 * NG), c = e % (4 * NG), n = min(n0 + c, width - 1), mr = min(m, rows - 1);
    float xs = 0.0f, gate[NB] = {};
    if (e < 16 * NG) {
        xs = x.p[(int64_t)mr * x.pitch + n];
        if (b0.gate.p) gate[0] = b0.gate.p[(int64_t)mr * b0.gate.pitch + n] + (b0.gate_bias ? b0.gate_bias[n] : 0.0f);
        if (NB > 1 && b1.gate.p) gate[NB - 1] = b1.gate.p[(int64_t)mr * b1.gate.pitch + n] + (b1.gate_bias ? b1.gate_bias[n] : 0.0f);
    }
    walk_branch<BF16, NG, WAVES, POLY0>(b0, rows, width, n0, s[0]);
    if (NB > 1) walk_branch<BF16, NG, WAVES, POLY1>(b1, rows, width, n0, s[NB - 1]);
#pragma unroll
    for (int b = 0; b < NB; b++) {
        const bool poly = b == 0 ? POLY0 : POLY1;
#pragma unroll
        for (int t = 0; t < 4; t++) {
            if (t > 0 && !poly) break;
#pragma unroll
            for (int g = 0; g < NG; g++) {
                f32x4 v;
#pragma unroll
                for (int r = 0; r < 4; r++) v[r] = blocks_sum(s[b].acc[g][t][r]);
                if (lane < 4) sums[b][wave][g][t][lane] = v;
            }
            if (t < 3 && poly) {
                const float q = blocks_sum(s[b].m[t]);
                if (lane < 4) squares[b][wave][t][lane] = q;
            }
        }
    }
    __syncthreads();
    if (e >= 16 * NG || m >= rows || n0 + c >= width) return;
#pragma unroll
    for (int b = 0; b < NB; b++) {
        const ResidualBranch &br = b == 0 ? b0 : b1;
        const bool poly = b == 0 ? POLY0 : POLY1;
        float y = 0.0f;
#pragma unroll
        for (int t = 0; t < 4; t++) {
            if (t > 0 && !poly) break;
            float v = 0.0f, q = 0.0f;
#pragma unroll
            for (int i = 0; i < WAVES; i++) v += sums[b][i][c / 4][t][m][c % 4];
            if (poly) {
                if (t < 3) {
#pragma unroll
                    for (int i = 0; i < WAVES; i++) q += squares[b][i][t][m];
                    v *= br.in.poly[t] / sqrtf(q / (float)br.in.k + br.in.eps);
                } else {
                    v *= br.in.poly[3];
                }
            }
            y += v;
        }
        xs += br.gate.p ? sigmoid(gate[b]) * y : y;
    }
    out[(int64_t)m * width + n0 + c] = xs;
}

// ---- many rows -------------------------------------------------------------------------------------------------------
__device__ __forceinline__ uint32_t round_bf16(float v) { return asu(v) + 0x7FFFu + ((asu(v) >> 16) & 1u); } // (bits above 15 hold the pattern)

// A workgroup per row: the row's sums, then the row as the product reads it.  FMT: 0 f32 words, 1 words rounded to
// bfloat16, 2 bfloat16 patterns.
template <int FMT> __global__ __launch_bounds__(kThreads) void product_input_kernel(const ProductInput in, void *__restrict__ dst) {
    __shared__ float red[kWaves];
    const uint32_t r = blockIdx.x;
    RowScale o;
    if (in.gamma || in.poly) {
        float m1 = 0.0f, m2 = 0.0f, m3 = 0.0f;
        for (uint32_t k = threadIdx.x; k < in.k; k += kThreads) {
            const float z = input_at(in, r, k), z2 = z * z;
            m1 += z2;
            if (in.poly) {
                m2 = fmaf(z2, z2, m2);
                m3 = fmaf(z2 * z2, z2, m3);
            }
        }
        m1 = block_sum(m1, red);
        if (in.poly) {
            m2 = block_sum(m2, red);
            m3 = block_sum(m3, red);
        }
        o = row_scale(in, m1, m2, m3);
    }
    const int64_t base = (int64_t)r * in.k;
    for (uint32_t k = threadIdx.x; k < in.k; k += kThreads) {
        const float v = scaled(in, o, input_at(in, r, k), k);
        if constexpr (FMT == 0) static_cast<float *>(dst)[base + k] = v;
        if constexpr (FMT == 1) static_cast<uint32_t *>(dst)[base + k] = round_bf16(v) & 0xFFFF0000u;
        if constexpr (FMT == 2) static_cast<uint16_t *>(dst)[base + k] = (uint16_t)(round_bf16(v) >> 16);
    }
}

// The same with every row held in registers between the two walks, four columns at a time: one part, k a multiple of 4,
// at most 4 * 256 * TRIPS columns.
template <int FMT, int TRIPS> __global__ __launch_bounds__(kThreads) void product_input_vec_kernel(const ProductInput in, void *__restrict__ dst) {
    __shared__ float red[kWaves];
    const uint32_t r = blockIdx.x;
    const float *x = in.x.p + (int64_t)r * in.x.pitch;
    float4 z[TRIPS];
    float m1 = 0.0f, m2 = 0.0f, m3 = 0.0f;
#pragma unroll
    for (int t = 0; t < TRIPS; t++) {
        const uint32_t k = (t * kThreads + threadIdx.x) * 4;
        z[t] = k < in.k ? *reinterpret_cast<const float4 *>(x + k) : make_float4(0.0f, 0.0f, 0.0f, 0.0f);
    }
    if (in.gamma || in.poly) {
#pragma unroll
        for (int t = 0; t < TRIPS; t++) {
            const float v[4] = {z[t].x, z[t].y, z[t].z, z[t].w};
#pragma unroll
            for (int j = 0; j < 4; j++) {
                const float z2 = v[j] * v[j];
                m1 += z2;
                if (in.poly) {
                    m2 = fmaf(z2, z2, m2);
                    m3 = fmaf(z2 * z2, z2, m3);
                }
            }
        }
        m1 = block_sum(m1, red);
        if (in.poly) {
            m2 = block_sum(m2, red);
            m3 = block_sum(m3, red);
        }
    }
    const RowScale o = row_scale(in, m1, m2, m3);
    const int64_t base = (int64_t)r * in.k;
#pragma unroll
    for (int t = 0; t < TRIPS; t++) {
        const uint32_t k = (t * kThreads + threadIdx.x) * 4;
        if (k >= in.k) continue;
        const float v[4] = {scaled(in, o, z[t].x, k), scaled(in, o, z[t].y, k + 1), scaled(in, o, z[t].z, k + 2), scaled(in, o, z[t].w, k + 3)};
        if constexpr (FMT == 0) *reinterpret_cast<float4 *>(static_cast<float *>(dst) + base + k) = make_float4(v[0], v[1], v[2], v[3]);
        if constexpr (FMT == 1)
            *reinterpret_cast<uint4 *>(static_cast<uint32_t *>(dst) + base + k) =
                make_uint4(round_bf16(v[0]) & 0xFFFF0000u, round_bf16(v[1]) & 0xFFFF0000u, round_bf16(v[2]) & 0xFFFF0000u, round_bf16(v[3]) & 0xFFFF0000u);
        if constexpr (FMT == 2)
            *reinterpret_cast<uint2 *>(static_cast<uint16_t *>(dst) + base + k) =
                make_uint2((round_bf16(v[0]) >> 16) | (round_bf16(v[1]) & 0xFFFF0000u), (round_bf16(v[2]) >> 16) | (round_bf16(v[3]) & 0xFFFF0000u));
    }
}

__global__ __launch_bounds__(kThreads) void affine_rows_kernel(float *__restrict__ y, const uint32_t n, const float *__restrict__ bias, const float scale) {
    const uint32_t k = blockIdx.x * kThreads + threadIdx.x;
    if (k >= n) return;
    float *p = y + (int64_t)blockIdx.y * n + k;
    *p = *p * scale + (bias ? bias[k] : 0.0f);
}

struct GatedSumArgs {
    Rows x;
    GatedTerm t[2];
    int n;
    uint32_t width;
    float scale;
    const void *extra; // [rows, slots, width]
    uint32_t slots;
    int extra_fmt;
};
template <int VW> __global__ __launch_bounds__(kThreads) void gated_sum_kernel(const GatedSumArgs a, float *__restrict__ out) {
    const uint32_t k = (blockIdx.x * kThreads + threadIdx.x) * VW, r = blockIdx.y;
    if (k >= a.width) return;
    float x[VW], s[VW] = {}, y[VW], g[VW];
    auto load = [&](const float *p, float(&v)[VW]) {
        if constexpr (VW == 4) {
            const float4 t = *reinterpret_cast<const float4 *>(p);
            v[0] = t.x, v[1] = t.y, v[2] = t.z, v[3] = t.w;
        } else {
            v[0] = *p;
        }
    };
    load(a.x.p + (int64_t)r * a.x.pitch + k, x);
#pragma unroll
    for (int i = 0; i < 2; i++) {
        if (i >= a.n) break;
        load(a.t[i].y + (int64_t)r * a.width + k, y);
        if (a.t[i].gate.p) load(a.t[i].gate.p + (int64_t)r * a.t[i].gate.pitch + k, g);
#pragma unroll
        for (int j = 0; j < VW; j++)
            s[j] += a.t[i].gate.p ? sigmoid(g[j] + (a.t[i].gate_bias ? a.t[i].gate_bias[k + j] : 0.0f)) * y[j] : y[j];
    }
    if (a.extra) {
#pragma unroll 4
        for (uint32_t i = 0; i < a.slots; i++) {
            const int64_t at = ((int64_t)r * a.slots + i) * a.width + k;
            if (a.extra_fmt == kFmtBF16) {
                const uint16_t *e = static_cast<const uint16_t *>(a.extra) + at;
                if constexpr (VW == 4) {
                    const uint2 t = *reinterpret_cast<const uint2 *>(e);
                    y[0] = bf16_lo(t.x), y[1] = bf16_hi(t.x), y[2] = bf16_lo(t.y), y[3] = bf16_hi(t.y);
                } else {
                    y[0] = asf((uint32_t)*e << 16);
                }
            } else {
                load(static_cast<const float *>(a.extra) + at, y);
            }
#pragma unroll
            for (int j = 0; j < VW; j++) s[j] += y[j];
        }
    }
#pragma unroll
    for (int j = 0; j < VW; j++) x[j] += a.scale * s[j];
    float *o = out + (int64_t)r * a.width + k;
    if constexpr (VW == 4) *reinterpret_cast<float4 *>(o) = make_float4(x[0], x[1], x[2], x[3]);
    else *o = x[0];
}

bool aligned16(const void *p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

int launched(const char *what) {
    const hipError_t e = hipGetLastError();
    return e == hipSuccess ? CG_OK : hip_fail(e, what);
}

// Kernels with more than 64 KB of dynamic LDS say so once.
template <class F> int allow_lds(F *kernel, size_t bytes) {
    if (bytes <= (64 << 10)) return CG_OK;
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, kFewRowsLds);
    return e == hipSuccess ? CG_OK : hip_fail(e, "hipFuncSetAttribute");
}

bool vector_rows(const Weight &w) {
    const int64_t vw = w.fmt == kFmtBF16 ? 8 : 4;
    return w.k % vw == 0 && w.pitch % vw == 0 && aligned16(w.p);
}

template <int M, int NC, bool BF16, bool VEC>
int few_rows_linear(cg_backend *be, const ProductInput &in, uint32_t rows, const Weight &w, const float *bias, float scale, float *out) {
    const uint32_t pitch = staged_pitch(in.k);
    const size_t bytes = (size_t)M * pitch * 4;
    if (int rc = allow_lds(few_rows_linear_kernel<M, NC, BF16, VEC>, bytes)) return rc;
    hipLaunchKernelGGL((few_rows_linear_kernel<M, NC, BF16, VEC>), dim3((w.n + kWaves * NC - 1) / (kWaves * NC)), dim3(kThreads), bytes, be->stream, in, rows, w,
                       pitch, bias, scale, out);
    return CG_OK;
}

template <int M, bool BF16, bool VEC, int NB>
int few_rows_residual(cg_backend *be, const Rows &x, const ResidualBranch *br, uint32_t rows, uint32_t width, float *out) {
    const uint32_t p0 = staged_pitch(br[0].in.k), p1 = NB > 1 ? staged_pitch(br[1].in.k) : 0;
    const size_t bytes = (size_t)M * (p0 + p1) * 4;
    if (int rc = allow_lds(few_rows_residual_kernel<M, BF16, VEC, NB>, bytes)) return rc;
    hipLaunchKernelGGL((few_rows_residual_kernel<M, BF16, VEC, NB>), dim3((width + kWaves - 1) / kWaves), dim3(kThreads), bytes, be->stream, x, br[0],
                       br[NB > 1 ? 1 : 0], rows, width, p0, p1, out);
    return CG_OK;
}

} // namespace

// The kernels for at most four rows read activations and weights 16 bytes at a time.
static bool four_rows(const ProductInput &in, uint32_t rows, const Weight &w) {
    const uint32_t vw = w.fmt == kFmtBF16 ? 8 : 4;
    return rows <= 4 && vector_rows(w) && in.k1 % vw == 0 && in.k % vw == 0 && in.x.pitch % 4 == 0 && aligned16(in.x.p) &&
           (!in.x2.p || (in.x2.pitch % 4 == 0 && aligned16(in.x2.p)));
}

static uint32_t column_groups(cg_backend *be, const Weight &w, uint32_t *iters) { // workgroups, which walk several groups when there are many
    const uint32_t groups = (w.n + 3) / 4, resident = (uint32_t)be->compute_units * 8;
    *iters = std::max(1u, (groups + resident - 1) / resident);
    return (groups + *iters - 1) / *iters;
}
template <bool BF16, int STEPS, int WAVES>
static void launch_four_rows(cg_backend *be, const ProductInput &in, uint32_t rows, const Weight &w, const float *bias, float scale, float *out) {
    uint32_t iters;
    const uint32_t blocks = column_groups(be, w, &iters);
    hipLaunchKernelGGL((four_rows_linear_kernel<BF16, STEPS, WAVES>), dim3(blocks), dim3(WAVES * 64), 0, be->stream, in, rows, w, iters, bias, scale, out);
}

int launch_few_rows_linear(cg_backend *be, const ProductInput &in, uint32_t rows, const Weight &w, const float *bias, float scale, float *out) {
    if (four_rows(in, rows, w) && !in.poly && in.k <= (w.fmt == kFmtBF16 ? 8192u : 4096u)) {
        const bool bf16 = w.fmt == kFmtBF16;
        ProfScope prof(be, CG_K_GEMM_SKINNY, (double)w.n * w.k * (bf16 ? 2.0 : 4.0) + 4.0 * rows * ((double)in.k + w.n));
        const uint32_t steps = (in.k + (bf16 ? 511 : 255)) / (bf16 ? 512 : 256); // of a workgroup of four waves
#define CG_FOUR(BF)                                                                              \
    if (steps <= 1) launch_four_rows<BF, 1, 4>(be, in, rows, w, bias, scale, out);               \
    else if (steps <= 2) launch_four_rows<BF, 2, 4>(be, in, rows, w, bias, scale, out);          \
    else if (steps <= 4) launch_four_rows<BF, 4, 4>(be, in, rows, w, bias, scale, out);          \
    else if (steps <= 8) launch_four_rows<BF, 4, 8>(be, in, rows, w, bias, scale, out);          \
    else launch_four_rows<BF, 8, 8>(be, in, rows, w, bias, scale, out)
        if (bf16) { CG_FOUR(true); }
        else { CG_FOUR(false); }
#undef CG_FOUR
        return launched("four_rows_linear");
    }
    const uint32_t m = few_rows_slots(rows, (uint64_t)staged_pitch(in.k) * 4);
    if (!m) return fail(CG_ERR_ARG, "internal error: too many rows for the streaming product");
    const bool bf16 = w.fmt == kFmtBF16, vec = vector_rows(w);
    ProfScope prof(be, CG_K_GEMM_SKINNY, (double)w.n * w.k * (bf16 ? 2.0 : 4.0) + 4.0 * rows * ((double)in.k + w.n));
    const int nc = !vec ? 1 : w.n >= 8192 ? 4 : w.n >= 4096 ? 2 : 1;
    int rc = CG_OK;
#define CG_LIN(M, NC, BF, VE) rc = few_rows_linear<M, NC, BF, VE>(be, in, rows, w, bias, scale, out)
#define CG_LIN_NC(M, BF)              \
    if (!vec) CG_LIN(M, 1, BF, false); \
    else if (nc == 4) CG_LIN(M, 4, BF, true); \
    else if (nc == 2) CG_LIN(M, 2, BF, true); \
    else CG_LIN(M, 1, BF, true)
#define CG_LIN_M(M)              \
    if (bf16) { CG_LIN_NC(M, true); } \
    else { CG_LIN_NC(M, false); }
    if (m == 1) { CG_LIN_M(1) }
    else if (m == 2) { CG_LIN_M(2) }
    else if (m == 4) { CG_LIN_M(4) }
    else { CG_LIN_M(8) }
#undef CG_LIN_M
#undef CG_LIN_NC
#undef CG_LIN
    return rc ? rc : launched("few_rows_linear");
}

template <bool BF16, int STEPS, int WAVES> static void launch_four_rows2(cg_backend *be, FourRowsJob (&j)[2], uint32_t rows) {
    const uint32_t b0 = column_groups(be, j[0].w, &j[0].iters), b1 = column_groups(be, j[1].w, &j[1].iters);
    hipLaunchKernelGGL((four_rows_linear2_kernel<BF16, STEPS, WAVES>), dim3(b0 + b1), dim3(WAVES * 64), 0, be->stream, j[0], j[1], b0, rows);
}

int launch_few_rows_linear2(cg_backend *be, const ProductInput (&in)[2], uint32_t rows, const Weight (&w)[2], float *const (&out)[2]) {
    const bool bf16 = w[0].fmt == kFmtBF16;
    FourRowsJob j[2];
    double bytes = 0.0;
    for (int i = 0; i < 2; i++) {
        if (!four_rows(in[i], rows, w[i]) || in[i].gamma || in[i].poly || w[i].fmt != w[0].fmt || in[i].k != in[0].k || in[i].k > (bf16 ? 8192u : 4096u)) return kDeclined;
        j[i] = {in[i], w[i], out[i], 1};
        bytes += (double)w[i].n * w[i].k * (bf16 ? 2.0 : 4.0) + 4.0 * rows * ((double)in[i].k + w[i].n);
    }
    ProfScope prof(be, CG_K_GEMM_SKINNY, bytes);
    const uint32_t steps = (in[0].k + (bf16 ? 511 : 255)) / (bf16 ? 512 : 256); // of a workgroup of four waves
#define CG_FOUR(BF)                                                  \
    if (steps <= 1) launch_four_rows2<BF, 1, 4>(be, j, rows);        \
    else if (steps <= 2) launch_four_rows2<BF, 2, 4>(be, j, rows);   \
    else if (steps <= 4) launch_four_rows2<BF, 4, 4>(be, j, rows);   \
    else if (steps <= 8) launch_four_rows2<BF, 4, 8>(be, j, rows);   \
    else launch_four_rows2<BF, 8, 8>(be, j, rows)
    if (bf16) { CG_FOUR(true); }
    else { CG_FOUR(false); }
#undef CG_FOUR
    return launched("four_rows_linear2");
}

template <bool BF16, int NG> static bool four_rows_residual(cg_backend *be, const Rows &x, const ResidualBranch *br, int n, uint32_t rows, uint32_t width, float *out) {
    constexpr int WAVES = 8;
    const dim3 grid((width + 4 * NG - 1) / (4 * NG)), block(WAVES * 64);
    const bool p0 = br[0].in.poly != nullptr, p1 = n > 1 && br[1].in.poly != nullptr;
    const ResidualBranch &b1 = br[n > 1 ? 1 : 0];
    hipStream_t s = be->stream;
    if (n == 2 && !p0 && p1) hipLaunchKernelGGL((four_rows_residual_kernel<BF16, 2, NG, WAVES, false, true>), grid, block, 0, s, x, br[0], b1, rows, width, out);
    else if (n == 2 && !p0 && !p1) hipLaunchKernelGGL((four_rows_residual_kernel<BF16, 2, NG, WAVES, false, false>), grid, block, 0, s, x, br[0], b1, rows, width, out);
    else if (n == 1 && p0) hipLaunchKernelGGL((four_rows_residual_kernel<BF16, 1, NG, WAVES, true, false>), grid, block, 0, s, x, br[0], b1, rows, width, out);
    else if (n == 1) hipLaunchKernelGGL((four_rows_residual_kernel<BF16, 1, NG, WAVES, false, false>), grid, block, 0, s, x, br[0], b1, rows, width, out);
    else return false;
    return true;
}

bool takes_few_rows_residual(const ResidualBranch *br, int n, uint32_t rows) {
    uint64_t per_row = 0;
    bool four = n > 0;
    for (int i = 0; i < n; i++) {
        per_row += (uint64_t)staged_pitch(br[i].in.k) * 4;
        four = four && four_rows(br[i].in, rows, br[i].w);
    }
    return n > 0 && (four || few_rows_slots(rows, per_row));
}

int launch_few_rows_residual(cg_backend *be, const Rows &x, const ResidualBranch *br, int n, uint32_t rows, uint32_t width, float *out) {
    bool four = n > 0 && (n == 1 || br[0].w.fmt == br[1].w.fmt) && !(n == 2 && br[0].in.poly);
    for (int i = 0; i < n; i++) four = four && four_rows(br[i].in, rows, br[i].w);
    if (four) {
        double work = 8.0 * rows * width;
        for (int i = 0; i < n; i++) work += (double)br[i].w.n * br[i].w.k * (br[i].w.fmt == kFmtBF16 ? 2.0 : 4.0) + 4.0 * rows * ((double)br[i].in.k + width);
        ProfScope prof(be, CG_K_GEMM_SKINNY, work);
        const bool bf16 = br[0].w.fmt == kFmtBF16, two = width >= (uint32_t)be->compute_units * 8;
        if (two) bf16 ? four_rows_residual<true, 2>(be, x, br, n, rows, width, out) : four_rows_residual<false, 2>(be, x, br, n, rows, width, out);
        else bf16 ? four_rows_residual<true, 1>(be, x, br, n, rows, width, out) : four_rows_residual<false, 1>(be, x, br, n, rows, width, out);
        return launched("four_rows_residual");
    }
    uint64_t per_row = 0;
    double bytes = 8.0 * rows * width;
    bool vec = true;
    for (int i = 0; i < n; i++) {
        per_row += (uint64_t)staged_pitch(br[i].in.k) * 4;
        bytes += (double)br[i].w.n * br[i].w.k * (br[i].w.fmt == kFmtBF16 ? 2.0 : 4.0) + 4.0 * rows * ((double)br[i].in.k + width);
        vec = vec && vector_rows(br[i].w);
    }
    const uint32_t m = few_rows_slots(rows, per_row);
    if (!m || n < 1) return fail(CG_ERR_ARG, "internal error: too many rows for the streaming product");
    ResidualBranch same[2] = {br[0], br[n > 1 ? 1 : 0]};
    if (n > 1 && same[0].w.fmt != same[1].w.fmt) { // one small matrix in words, the other in patterns: one branch after the other
        if (int rc = launch_few_rows_residual(be, x, br, 1, rows, width, out)) return rc;
        Rows o{out, (int64_t)width};
        return launch_few_rows_residual(be, o, br + 1, 1, rows, width, out);
    }
    const bool bf16 = br[0].w.fmt == kFmtBF16;
    ProfScope prof(be, CG_K_GEMM_SKINNY, bytes);
    int rc = CG_OK;
#define CG_RES(M, BF, VE)                                                                       \
    rc = n > 1 ? few_rows_residual<M, BF, VE, 2>(be, x, same, rows, width, out) : few_rows_residual<M, BF, VE, 1>(be, x, same, rows, width, out)
#define CG_RES_M(M)                       \
    if (bf16 && vec) CG_RES(M, true, true);       \
    else if (bf16) CG_RES(M, true, false);        \
    else if (vec) CG_RES(M, false, true);         \
    else CG_RES(M, false, false)
    if (m == 1) { CG_RES_M(1); }
    else if (m == 2) { CG_RES_M(2); }
    else if (m == 4) { CG_RES_M(4); }
    else { CG_RES_M(8); }
#undef CG_RES_M
#undef CG_RES
    return rc ? rc : launched("few_rows_residual");
}

int launch_product_input(cg_backend *be, const ProductInput &in, uint32_t rows, void *dst, bool round_bf16, int fmt) {
    ProfScope prof(be, CG_K_REDUCE, (double)rows * in.k * (4.0 + (fmt == kFmtBF16 ? 2.0 : 4.0)));
    const int f = fmt == kFmtBF16 ? 2 : round_bf16 ? 1 : 0;
    const bool vec = !in.x2.p && in.k % 4 == 0 && in.x.pitch % 4 == 0 && aligned16(in.x.p) && in.k <= 4 * kThreads * 16;
    const int trips = (int)((in.k + 4 * kThreads - 1) / (4 * kThreads));
    hipStream_t s = be->stream;
#define CG_IN(F)                                                                                                                       \
    if (!vec) hipLaunchKernelGGL((product_input_kernel<F>), dim3(rows), dim3(kThreads), 0, s, in, dst);                                 \
    else if (trips <= 1) hipLaunchKernelGGL((product_input_vec_kernel<F, 1>), dim3(rows), dim3(kThreads), 0, s, in, dst);               \
    else if (trips <= 2) hipLaunchKernelGGL((product_input_vec_kernel<F, 2>), dim3(rows), dim3(kThreads), 0, s, in, dst);               \
    else if (trips <= 4) hipLaunchKernelGGL((product_input_vec_kernel<F, 4>), dim3(rows), dim3(kThreads), 0, s, in, dst);               \
    else if (trips <= 8) hipLaunchKernelGGL((product_input_vec_kernel<F, 8>), dim3(rows), dim3(kThreads), 0, s, in, dst);               \
    else hipLaunchKernelGGL((product_input_vec_kernel<F, 16>), dim3(rows), dim3(kThreads), 0, s, in, dst)
    if (f == 0) { CG_IN(0); }
    else if (f == 1) { CG_IN(1); }
    else { CG_IN(2); }
#undef CG_IN
    return launched("product_input");
}

int launch_affine_rows(cg_backend *be, float *y, uint32_t rows, uint32_t n, const float *bias, float scale) {
    for (uint32_t r0 = 0; r0 < rows; r0 += 65535) { // (the grid's y extent)
        const uint32_t nr = rows - r0 < 65535 ? rows - r0 : 65535;
        ProfScope prof(be, CG_K_ELEMENTWISE, 8.0 * nr * n);
        hipLaunchKernelGGL(affine_rows_kernel, dim3((n + kThreads - 1) / kThreads, nr), dim3(kThreads), 0, be->stream, y + (int64_t)r0 * n, n, bias, scale);
    }
    return launched("affine_rows");
}

int launch_gated_sum(cg_backend *be, const Rows &x, const GatedTerm *t, int n, uint32_t rows, uint32_t width, float *out, float scale, const void *extra,
                     uint32_t slots, int extra_fmt) {
    bool vec = width % 4 == 0 && x.pitch % 4 == 0 && aligned16(x.p) && aligned16(out) && aligned16(extra);
    for (int i = 0; i < n; i++) vec = vec && (!t[i].gate.p || (t[i].gate.pitch % 4 == 0 && aligned16(t[i].gate.p))) && aligned16(t[i].y);
    for (uint32_t r0 = 0; r0 < rows; r0 += 65535) {
        const uint32_t nr = rows - r0 < 65535 ? rows - r0 : 65535;
        ProfScope prof(be, CG_K_ELEMENTWISE, (2.0 + 2.0 * n + (extra ? (extra_fmt == kFmtBF16 ? 0.5 : 1.0) * slots : 0.0)) * 4.0 * nr * width);
        GatedSumArgs a{};
        a.x = {x.p + (int64_t)r0 * x.pitch, x.pitch};
        a.n = n;
        a.width = width;
        a.scale = scale;
        a.extra = extra ? static_cast<const char *>(extra) + (int64_t)r0 * slots * width * (extra_fmt == kFmtBF16 ? 2 : 4) : nullptr;
        a.slots = slots;
        a.extra_fmt = extra_fmt;
        for (int i = 0; i < n; i++) {
            a.t[i] = t[i];
            a.t[i].y += (int64_t)r0 * width;
            if (a.t[i].gate.p) a.t[i].gate.p += (int64_t)r0 * a.t[i].gate.pitch;
        }
        const uint32_t per = kThreads * (vec ? 4 : 1);
        const dim3 grid((width + per - 1) / per, nr);
        if (vec) hipLaunchKernelGGL((gated_sum_kernel<4>), grid, dim3(kThreads), 0, be->stream, a, out + (int64_t)r0 * width);
        else hipLaunchKernelGGL((gated_sum_kernel<1>), grid, dim3(kThreads), 0, be->stream, a, out + (int64_t)r0 * width);
    }
    return launched("gated_sum");
}

} // namespace cg
