// What stands around a decoder layer's products: embeddings of tokens and token pairs, grouped norms with short filters over
// time, and the vectors that tokens add to their rows.
#include "block_stream.hpp"

#include <algorithm>

namespace cg {
namespace {

constexpr int kThreads = 256, kWaves = 4;

__device__ __forceinline__ uint32_t round_bf16(float v) { return asu(v) + 0x7FFFu + ((asu(v) >> 16) & 1u); } // (bits above 15 hold the pattern)
__device__ __forceinline__ float element(const Table &t, int64_t i) {
    return t.fmt == kFmtBF16 ? asf((uint32_t)static_cast<const uint16_t *>(t.p)[i] << 16) : static_cast<const float *>(t.p)[i];
}
__device__ __forceinline__ uint32_t token_at(const Tokens &t, uint32_t r) { return t.p ? t.p[r] : t.value; }

// ---- embeddings ------------------------------------------------------------------------------------------------------
// a workgroup per token
__global__ __launch_bounds__(kThreads) void pair_embedding_kernel(const PairEmbeddingPlan p, uint32_t *fault) {
    const uint32_t r = blockIdx.x, b = r / p.S, s = r - b * p.S;
    uint32_t id = token_at(p.ids, r), before = 0;
    const bool first = s == 0 && !p.previous_n;
    if (s) before = token_at(p.ids, r - 1);
    else if (!first) before = p.previous.p ? p.previous.p[(b + 1) * p.previous_n - 1] : p.previous.value;
    if (threadIdx.x == 0 && s + 1 == p.S) p.previous_out[b] = id;
    if (id >= p.vocab) {
        if (threadIdx.x == 0) *fault = kFaultIndexRange;
        id = 0;
    }
    // (the multipliers are taken modulo the buckets already: no overflow)
    const uint64_t pair = ((uint64_t)before * p.mul_prev % p.buckets + (uint64_t)id * p.mul_cur % p.buckets) % p.buckets;
    const int64_t a = (int64_t)id * p.table.pitch, c = (int64_t)(first ? p.buckets : pair) * p.pairs.pitch;
    for (uint32_t k = threadIdx.x; k < p.width; k += kThreads) p.out[(int64_t)r * p.width + k] = element(p.table, a + k) + element(p.pairs, c + k);
}

// ---- grouped norm and filter -----------------------------------------------------------------------------------------
// A workgroup takes `run` tokens of a sequence and `cols` columns of a group (blockIdx.y: group and part of it): the scales of
// these tokens' rows and of the taps - 1 before them (a wave per row, four rows' pieces in flight), then, with a thread per VW
// columns, the filter along the tokens; what the filter looks back on stays in registers.  TAPS: at most so many.
template <int VW, int TAPS> __global__ __launch_bounds__(kThreads) void conv_rows_kernel(const ConvRowsPlan p, const uint32_t parts) {
    extern __shared__ float scale[]; // [run + taps - 1]
    const uint32_t past = p.taps - 1, size = p.width / p.groups, group = blockIdx.y / parts, part = blockIdx.y - group * parts, g0 = group * size;
    const uint32_t runs = (p.S + p.run - 1) / p.run, b = blockIdx.x / runs, s0 = (blockIdx.x - b * runs) * p.run, n = min(p.run, p.S - s0);
    const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    auto load = [&](const float *q, float(&v)[VW]) {
        if constexpr (VW == 4) {
            const float4 t = *reinterpret_cast<const float4 *>(q);
            v[0] = t.x, v[1] = t.y, v[2] = t.z, v[3] = t.w;
        } else {
            v[0] = *q;
        }
    };
    // this thread's columns, its share of the filters asked for first
    const uint32_t per = ((size + parts - 1) / parts + VW - 1) / VW * VW, c_end = g0 + min(size, (part + 1) * per);
    // few columns: the workgroup's waves take parts of the run
    const uint32_t across = min(kThreads, ((per + VW - 1) / VW + 63) / 64 * 64), subs = kThreads / across, sub = threadIdx.x / across;
    const uint32_t sub_run = (n + subs - 1) / subs, i_first = min(n, sub * sub_run), i_end = min(n, i_first + sub_run);
    const uint32_t c_first = g0 + part * per + (threadIdx.x - sub * across) * VW;
    float gamma[2][VW], w[2][TAPS][VW]; // tap t counts from the present back
    auto ask_filters = [&](uint32_t at) {
        at = min(at, p.width - VW);
#pragma unroll
        for (int f = 0; f < 2; f++) {
            if (f >= p.n) break;
            load(p.out[f].gamma + at, gamma[f]);
#pragma unroll
            for (int j = 0; j < VW; j++) {
                if (TAPS == 4 && VW == 4 && p.taps == 4 && p.out[f].conv) {
                    const float4 t = *reinterpret_cast<const float4 *>(p.out[f].conv + (int64_t)(at + j) * 4);
                    w[f][0][j] = t.w, w[f][1 % TAPS][j] = t.z, w[f][2 % TAPS][j] = t.y, w[f][3 % TAPS][j] = t.x;
                } else {
#pragma unroll
                    for (int t = 0; t < TAPS; t++) w[f][t][j] = p.out[f].conv && t < (int)p.taps ? p.out[f].conv[(int64_t)(at + j) * p.taps + (p.taps - 1 - t)] : 0.0f;
                }
            }
        }
    };
    ask_filters(c_first);
    constexpr int ROWS = 4; // of a wave at a time
    for (uint32_t i0 = wave; i0 < n + past; i0 += kWaves * ROWS) {
        float m[ROWS] = {};
        for (uint32_t k = lane * VW; k < size; k += 64 * VW) {
            float v[ROWS][VW];
#pragma unroll
            for (int e = 0; e < ROWS; e++) { // (clamped: rows that are not there are not stored)
                const int32_t s = (int32_t)(s0 + min(i0 + e * kWaves, n + past - 1)) - (int32_t)past;
                load(p.x.p + ((int64_t)b * p.S + max(s, 0)) * p.x.pitch + g0 + k, v[e]);
            }
#pragma unroll
            for (int e = 0; e < ROWS; e++)
#pragma unroll
                for (int j = 0; j < VW; j++) m[e] = fmaf(v[e][j], v[e][j], m[e]);
        }
#pragma unroll
        for (int e = 0; e < ROWS; e++) {
            const uint32_t i = i0 + e * kWaves;
            const float sum = wave_total(m[e]);
            if (lane == 0 && i < n + past) scale[i] = 1.0f / sqrtf(sum / (float)size + p.eps);
        }
    }
    __syncthreads();
    if (sub >= subs || i_first == i_end) return;
    for (uint32_t c = c_first; c < c_end; c += across * VW) {
        if (c != c_first) ask_filters(c);
        // z of token s0 - past + i, for the tokens in front of the sequence's new ones from its state
        auto unit = [&](uint32_t i, float(&v)[VW]) {
            const int32_t s = (int32_t)(s0 + i) - (int32_t)past;
            if (s >= 0) {
                load(p.x.p + ((int64_t)b * p.S + s) * p.x.pitch + c, v);
#pragma unroll
                for (int j = 0; j < VW; j++) v[j] *= scale[i];
            } else if (p.state) {
                load(p.state + ((int64_t)b * past + (past + s)) * p.width + c, v);
            } else {
#pragma unroll
                for (int j = 0; j < VW; j++) v[j] = 0.0f;
            }
        };
        // the inputs behind the sequence's end become its state
        auto keep = [&](int32_t s, const float(&v)[VW]) {
            const int32_t at = s - ((int32_t)p.S - (int32_t)past);
            if (at < 0) return;
            float *o = p.state_out + ((int64_t)b * past + at) * p.width + c;
            if constexpr (VW == 4) *reinterpret_cast<float4 *>(o) = make_float4(v[0], v[1], v[2], v[3]);
            else *o = v[0];
        };
        float z[TAPS][VW]; // the input t tokens back
#pragma unroll
        for (int t = 0; t < TAPS; t++)
#pragma unroll
            for (int j = 0; j < VW; j++) z[t][j] = 0.0f;
#pragma unroll
        for (int t = TAPS - 1; t >= 1; t--)
            if (t <= (int)past) {
                const int32_t s = (int32_t)(s0 + i_first) - t;
                unit(past + i_first - t, z[t - 1]); // (moved one back below)
                if (s0 + i_end == p.S && s < 0) keep(s, z[t - 1]);
            }
        constexpr int AHEAD = 4; // rows asked for together
        for (uint32_t i0 = i_first; i0 < i_end; i0 += AHEAD) {
            float next[AHEAD][VW];
#pragma unroll
            for (int e = 0; e < AHEAD; e++) unit(past + min(i0 + e, i_end - 1), next[e]);
#pragma unroll
            for (int e = 0; e < AHEAD; e++) {
                const uint32_t s = s0 + i0 + e;
                if (i0 + e >= i_end) break;
#pragma unroll
                for (int t = TAPS - 1; t >= 1; t--)
#pragma unroll
                    for (int j = 0; j < VW; j++) z[t][j] = z[t - 1][j];
#pragma unroll
                for (int j = 0; j < VW; j++) z[0][j] = next[e][j];
                if (past) keep((int32_t)s, z[0]);
                const int64_t o = ((int64_t)b * p.S + s) * p.width + c;
#pragma unroll
                for (int f = 0; f < 2; f++) {
                    if (f >= p.n) break;
                    float h[VW];
#pragma unroll
                    for (int j = 0; j < VW; j++) {
                        float a = 0.0f;
#pragma unroll
                        for (int t = TAPS - 1; t >= 0; t--) a = fmaf(w[f][t][j], z[t][j], a);
                        h[j] = (a + z[0][j]) * gamma[f][j];
                    }
                    if (p.out[f].fmt == kFmtBF16) {
                        uint16_t *d = static_cast<uint16_t *>(p.out[f].dst) + o;
                        if constexpr (VW == 4)
                            *reinterpret_cast<uint2 *>(d) =
                                make_uint2((round_bf16(h[0]) >> 16) | (round_bf16(h[1]) & 0xFFFF0000u), (round_bf16(h[2]) >> 16) | (round_bf16(h[3]) & 0xFFFF0000u));
                        else *d = (uint16_t)(round_bf16(h[0]) >> 16);
                    } else {
                        float *d = static_cast<float *>(p.out[f].dst) + o;
                        if (p.out[f].round) {
#pragma unroll
                            for (int j = 0; j < VW; j++) h[j] = asf(round_bf16(h[j]) & 0xFFFF0000u);
                        }
                        if constexpr (VW == 4) *reinterpret_cast<float4 *>(d) = make_float4(h[0], h[1], h[2], h[3]);
                        else *d = h[0];
                    }
                }
            }
        }
    }
}

// ---- the tokens' own vectors -----------------------------------------------------------------------------------------
__device__ __forceinline__ float gelu(float v) { // 1 + tanh(t) = 2 / (1 + e^(-2 t))
    const float t = 0.79788456080286536f * (v + 0.044715f * v * v * v);
    return v / (1.0f + expf(-2.0f * t));
}

// g[r, i] = gelu(g[r, i]) * table[id_r, first + i], in place
__global__ __launch_bounds__(kThreads) void side_gate_kernel(float *__restrict__ g, const Tokens ids, const Table table, const uint32_t vocab, const uint32_t first,
                                                             const uint32_t dim, const uint32_t rows, uint32_t *fault) {
    const uint64_t i = (uint64_t)blockIdx.x * kThreads + threadIdx.x;
    if (i >= (uint64_t)rows * dim) return;
    const uint32_t r = (uint32_t)(i / dim), k = (uint32_t)(i - (uint64_t)r * dim);
    uint32_t id = token_at(ids, r);
    if (id >= vocab) {
        *fault = kFaultIndexRange;
        id = 0;
    }
    g[i] = gelu(g[i]) * element(table, (int64_t)id * table.pitch + first + k);
}

// The same for a few rows with the product in front: a wave per (row, value).
template <bool BF16, bool VEC>
__global__ __launch_bounds__(kThreads) void side_first_kernel(const Rows x, const Weight w, const Tokens ids, const Table table, const uint32_t vocab, const uint32_t first,
                                                              float *__restrict__ g, uint32_t *fault) {
    typedef Streamed<BF16, VEC> St;
    constexpr uint32_t W = St::W, SPAN = 64 * W, EB = BF16 ? 2 : 4;
    const uint32_t lane = threadIdx.x & 63, i = blockIdx.x * kWaves + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), r = blockIdx.y;
    if (i >= w.n) return;
    uint32_t id = token_at(ids, r);
    if (id >= vocab) {
        *fault = kFaultIndexRange;
        id = 0;
    }
    const float e = element(table, (int64_t)id * table.pitch + first + i);
    const char *row = static_cast<const char *>(w.p) + (int64_t)i * w.pitch * EB;
    const float *xr = x.p + (int64_t)r * x.pitch;
    float a = 0.0f;
#pragma unroll 4
    for (uint32_t k = lane * W; k < w.k; k += SPAN) {
        St s;
        s.load(row, k);
        float v[W];
        St::input(xr, k, v);
        a = s.dot(v, a);
    }
    a = wave_total(a);
    if (lane == 0) g[(int64_t)r * w.n + i] = gelu(a) * e;
}

// The rest for a few rows in one launch, a workgroup per row: LANES lanes share a row of w (all of it in 16-byte pieces), its
// product with g ends in the last of them, and stays there until the row's mean square is known.  WORK: rows of w per LANES lanes.
constexpr int kSideThreads = 1024;
template <bool BF16, int LANES, int WORK>
__global__ __launch_bounds__(kSideThreads) void side_second_kernel(const Rows x, const float *__restrict__ g, const Weight w, const float *__restrict__ norm, const float eps,
                                                                   const float scale, float *__restrict__ out) {
    typedef Streamed<BF16, true> St;
    constexpr uint32_t W = St::W, EB = BF16 ? 2 : 4, PER = kSideThreads / LANES;
    __shared__ float red[kSideThreads / 64];
    const uint32_t sub = threadIdx.x % LANES, n0 = threadIdx.x / LANES, k = min(sub * W, w.k - W);
    const int64_t r = blockIdx.x;
    St s[WORK];
#pragma unroll
    for (int i = 0; i < WORK; i++) s[i].load(static_cast<const char *>(w.p) + (int64_t)min(n0 + i * PER, w.n - 1) * w.pitch * EB, k);
    float v[W], y[WORK], m = 0.0f;
    St::input(g + r * w.k, k, v);
#pragma unroll
    for (uint32_t j = 0; j < W; j++) v[j] = sub * W < w.k ? v[j] : 0.0f;
#pragma unroll
    for (int i = 0; i < WORK; i++) {
        float a = s[i].dot(v, 0.0f);
        if (LANES >= 2) a = add_shifted<0x111, 0xF>(a);
        if (LANES >= 4) a = add_shifted<0x112, 0xF>(a);
        if (LANES >= 8) a = add_shifted<0x114, 0xF>(a);
        if (LANES >= 16) a = add_shifted<0x118, 0xF>(a);
        y[i] = a;
        if (sub == LANES - 1 && n0 + i * PER < w.n) m = fmaf(a, a, m);
    }
    m = wave_total(m);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = m;
    __syncthreads();
    m = 0.0f;
#pragma unroll
    for (int i = 0; i < kSideThreads / 64; i++) m += red[i];
    const float f = scale / sqrtf(m / (float)w.n + eps);
    if (sub != LANES - 1) return;
#pragma unroll
    for (int i = 0; i < WORK; i++) {
        const uint32_t n = n0 + i * PER;
        if (n < w.n) out[r * w.n + n] = fmaf(y[i] * f, norm[n], x.p[r * x.pitch + n]);
    }
}

// out = x + scale * y / sqrt(mean(y^2) + eps) * norm; a workgroup per row
template <int VW> __global__ __launch_bounds__(kThreads) void side_sum_kernel(const Rows x, const float *__restrict__ y, const float *__restrict__ norm, const uint32_t width,
                                                                             const float eps, const float scale, float *__restrict__ out) {
    __shared__ float red[kWaves];
    const int64_t r = blockIdx.x;
    const float *yr = y + r * width, *xr = x.p + r * x.pitch;
    auto load = [&](const float *q, float(&v)[VW]) {
        if constexpr (VW == 4) {
            const float4 t = *reinterpret_cast<const float4 *>(q);
            v[0] = t.x, v[1] = t.y, v[2] = t.z, v[3] = t.w;
        } else {
            v[0] = *q;
        }
    };
    float m = 0.0f;
    for (uint32_t k = threadIdx.x * VW; k < width; k += kThreads * VW) {
        float v[VW];
        load(yr + k, v);
#pragma unroll
        for (int j = 0; j < VW; j++) m = fmaf(v[j], v[j], m);
    }
    m = wave_total(m);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = m;
    __syncthreads();
    const float f = scale / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)width + eps);
    for (uint32_t k = threadIdx.x * VW; k < width; k += kThreads * VW) {
        float v[VW], xs[VW], w[VW];
        load(yr + k, v);
        load(xr + k, xs);
        load(norm + k, w);
#pragma unroll
        for (int j = 0; j < VW; j++) xs[j] = fmaf(v[j] * f, w[j], xs[j]);
        float *o = out + r * width + k;
        if constexpr (VW == 4) *reinterpret_cast<float4 *>(o) = make_float4(xs[0], xs[1], xs[2], xs[3]);
        else *o = xs[0];
    }
}

bool aligned16(const void *p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

int launched(const char *what) {
    const hipError_t e = hipGetLastError();
    return e == hipSuccess ? CG_OK : hip_fail(e, what);
}

} // namespace

int launch_pair_embedding(cg_backend *be, const PairEmbeddingPlan &p) {
    ProfScope prof(be, CG_K_GATHER, (double)p.B * p.S * p.width * (4.0 + 2.0 * (p.table.fmt == kFmtBF16 ? 2.0 : 4.0)));
    hipLaunchKernelGGL(pair_embedding_kernel, dim3(p.B * p.S), dim3(kThreads), 0, be->stream, p, be->fault_dev);
    return launched("pair_embedding");
}

int launch_conv_rows(cg_backend *be, ConvRowsPlan p) {
    const uint32_t cols = p.width / p.groups, past = p.taps - 1;
    // short runs while the device is not full, and a group's columns over several workgroups
    p.run = 1;
    while (p.run < 16 && (uint64_t)p.B * p.groups * ((p.S + p.run * 2 - 1) / (p.run * 2)) >= 8ull * be->compute_units) p.run *= 2;
    uint32_t split = 1;
    while (cols / (split * 2) >= 128 && (uint64_t)p.B * p.S * p.groups * split * 2 <= be->compute_units) split *= 2;
    double bytes = 4.0;
    bool vec = cols % 4 == 0 && p.x.pitch % 4 == 0 && aligned16(p.x.p) && aligned16(p.state) && aligned16(p.state_out);
    for (int f = 0; f < p.n; f++) {
        bytes += p.out[f].fmt == kFmtBF16 ? 2.0 : 4.0;
        vec = vec && aligned16(p.out[f].dst) && aligned16(p.out[f].gamma) && aligned16(p.out[f].conv);
    }
    ProfScope prof(be, CG_K_REDUCE, bytes * p.B * p.S * p.width);
    const uint32_t runs = (p.S + p.run - 1) / p.run;
    const dim3 grid(p.B * runs, p.groups * split);
    const size_t lds = (p.run + past) * 4;
    hipStream_t s = be->stream;
#define CG_CONV(T)                                                                                       \
    if (vec) hipLaunchKernelGGL((conv_rows_kernel<4, T>), grid, dim3(kThreads), lds, s, p, split);        \
    else hipLaunchKernelGGL((conv_rows_kernel<1, T>), grid, dim3(kThreads), lds, s, p, split)
    if (p.taps <= 1) { CG_CONV(1); }
    else if (p.taps <= 2) { CG_CONV(2); }
    else if (p.taps <= 3) { CG_CONV(3); }
    else if (p.taps <= 4) { CG_CONV(4); }
    else if (p.taps <= 8) { CG_CONV(8); }
    else if (p.taps <= kMaxTaps) { CG_CONV(kMaxTaps); }
    else return fail(CG_ERR_UNSUPPORTED, "block_conv_linear: at most %u taps", kMaxTaps);
#undef CG_CONV
    return launched("conv_rows");
}

int launch_side_gate(cg_backend *be, float *g, const Tokens &ids, const Table &table, uint32_t vocab, uint32_t first, uint32_t dim, uint32_t rows) {
    ProfScope prof(be, CG_K_ELEMENTWISE, 12.0 * rows * dim);
    const uint64_t n = (uint64_t)rows * dim;
    hipLaunchKernelGGL(side_gate_kernel, dim3((uint32_t)((n + kThreads - 1) / kThreads)), dim3(kThreads), 0, be->stream, g, ids, table, vocab, first, dim, rows,
                       be->fault_dev);
    return launched("side_gate");
}

int launch_side_first(cg_backend *be, const Rows &x, uint32_t rows, const Weight &w, const Tokens &ids, const Table &table, uint32_t vocab, uint32_t first, float *g) {
    const bool bf16 = w.fmt == kFmtBF16;
    const uint32_t vw = bf16 ? 8 : 4;
    const bool vec = w.k % vw == 0 && w.pitch % vw == 0 && aligned16(w.p) && x.pitch % 4 == 0 && aligned16(x.p);
    ProfScope prof(be, CG_K_GEMM_SKINNY, (double)w.n * w.k * (bf16 ? 2.0 : 4.0) + 4.0 * rows * ((double)w.k + w.n));
    const dim3 grid((w.n + kWaves - 1) / kWaves, rows);
#define CG_FIRST(BF, VE) hipLaunchKernelGGL((side_first_kernel<BF, VE>), grid, dim3(kThreads), 0, be->stream, x, w, ids, table, vocab, first, g, be->fault_dev)
    if (bf16 && vec) CG_FIRST(true, true);
    else if (bf16) CG_FIRST(true, false);
    else if (vec) CG_FIRST(false, true);
    else CG_FIRST(false, false);
#undef CG_FIRST
    return launched("side_first");
}

template <bool BF16, int LANES> static int side_second(cg_backend *be, const Rows &x, const float *g, uint32_t rows, const Weight &w, const float *norm, float eps, float scale, float *out) {
    const uint32_t work = (w.n + kSideThreads / LANES - 1) / (kSideThreads / LANES);
#define CG_SECOND(WK) hipLaunchKernelGGL((side_second_kernel<BF16, LANES, WK>), dim3(rows), dim3(kSideThreads), 0, be->stream, x, g, w, norm, eps, scale, out)
    if (work <= 4) CG_SECOND(4);
    else if (work <= 8) CG_SECOND(8);
    else if (work <= 16) CG_SECOND(16);
    else return kDeclined;
#undef CG_SECOND
    return launched("side_second");
}

constexpr uint64_t kSideBytes = 64 << 10; // of a matrix that one compute unit reads sooner than two launches pass

int launch_side_second(cg_backend *be, const Rows &x, const float *g, uint32_t rows, const Weight &w, const float *norm, float eps, float scale, float *out) {
    const bool bf16 = w.fmt == kFmtBF16;
    const uint32_t vw = bf16 ? 8 : 4, pieces = (w.k + vw - 1) / vw;
    if (w.k % vw || w.pitch % vw || !aligned16(w.p) || !aligned16(g) || pieces > 16 || (uint64_t)w.n * w.k * (bf16 ? 2 : 4) > kSideBytes) return kDeclined;
    ProfScope prof(be, CG_K_GEMM_SKINNY, (double)w.n * w.k * (bf16 ? 2.0 : 4.0) + 4.0 * rows * ((double)w.k + 2.0 * w.n));
#define CG_SIDE(L) return bf16 ? side_second<true, L>(be, x, g, rows, w, norm, eps, scale, out) : side_second<false, L>(be, x, g, rows, w, norm, eps, scale, out)
    if (pieces <= 1) CG_SIDE(1);
    if (pieces <= 2) CG_SIDE(2);
    if (pieces <= 4) CG_SIDE(4);
    if (pieces <= 8) CG_SIDE(8);
    CG_SIDE(16);
#undef CG_SIDE
}

int launch_side_sum(cg_backend *be, const Rows &x, const float *y, const float *norm, uint32_t rows, uint32_t width, float eps, float scale, float *out) {
    ProfScope prof(be, CG_K_REDUCE, 12.0 * rows * width);
    const bool vec = width % 4 == 0 && x.pitch % 4 == 0 && aligned16(x.p) && aligned16(y) && aligned16(norm) && aligned16(out);
    if (vec) hipLaunchKernelGGL((side_sum_kernel<4>), dim3(rows), dim3(kThreads), 0, be->stream, x, y, norm, width, eps, scale, out);
    else hipLaunchKernelGGL((side_sum_kernel<1>), dim3(rows), dim3(kThreads), 0, be->stream, x, y, norm, width, eps, scale, out);
    return launched("side_sum");
}

} // namespace cg
