// cg_block_attention for more than a few new tokens: 16 query rows of all heads against 16 keys at a time, every product on
// v_mfma_f32_16x16x4.  Head mixing after the soft-max needs the finished weights of every head for the same (query, key),
// so the rows' sums come first, from a launch of their own:
//
//   attention_row_stats_kernel  a wave per (16 query rows, one or two heads): a bound on every row's scores and the sum of its exponentials
//   attention_tiles_kernel      8 waves per 16 query rows, a few heads each: scores again, weights to LDS, mixed there over
//                               the heads (as the product talk . weights, a column per (query, key)), times the values.
//                               The three run a key tile apart from each other on three buffers, so that one barrier per
//                               key tile is enough and what one waits for is covered by the other two.  The keys of a row
//                               tile may be cut over several workgroups: finished weights only add up.
//
// The 16x16x4 instruction takes A[i = lane % 16][k = lane / 16], B[k = lane / 16][j = lane % 16] and leaves
// C[4 (lane / 16) + r][lane % 16] in register r.  The order of k inside a product is free: lane group g supplies
// k = 16 c + 4 g + t to the t-th of four instructions, for A and B alike, so an operand that is contiguous along k is read
// 16 bytes at a time.
#include "blocks.hpp"
#include "device_utils.hpp"

#include <algorithm>

namespace cg {
namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));

constexpr int kTileWaves = 8, kStatWaves = 4;
constexpr uint32_t kRowsT = 16, kKeysT = 16;
constexpr uint32_t kRowPitch = kKeysT + 4;                // floats; 16-byte reads of 16 rows cover all banks
constexpr uint32_t kHeadPitch = kRowsT * kRowPitch + 4;   // heads four apart lie 16 banks apart
constexpr float kLog2e = 1.44269504088896341f;

__device__ __forceinline__ f32x4 mfma(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
__device__ __forceinline__ float slope_of(uint32_t h, uint32_t heads) { return exp2f(-8.0f * (float)(h + 1) / (float)heads); }

// Workgroup ids go to the eight XCDs in turn, each with an L2 of its own: runs of 16 row tiles, which read nearly the same
// keys, are given to one XCD when a window makes nearly all of them the same work.  n: row tiles of a sequence; the last
// rows, which see the most keys, go first.
__device__ __forceinline__ uint32_t tile_of(const AttentionPlan &p, uint32_t id, uint32_t n) {
    constexpr uint32_t kRun = 16, kXcds = 8;
    const uint32_t whole = p.window && p.window <= p.S / 4 ? n / (kRun * kXcds) * (kRun * kXcds) : 0;
    if (id < whole) {
        const uint32_t slot = id / kXcds, xcd = id % kXcds;
        id = (slot / kRun * kXcds + xcd) * kRun + slot % kRun;
    }
    return n - 1 - id;
}

// What a wave knows of its place: query rows s0 .. s0 + 15 of sequence b, lane (li, lg).
struct Place {
    uint32_t b, s0, li, lg;
};

// The first and one past the last key that any of the tile's rows sees.
__device__ __forceinline__ void tile_keys(const AttentionPlan &p, uint32_t s0, uint32_t *lo, uint32_t *hi) {
    const uint32_t first = p.cached + s0, last = p.cached + min(s0 + kRowsT, p.S) - 1;
    *lo = p.window && first + 1 > p.window ? first + 1 - p.window : 0;
    *hi = last + 1;
}

template <int DT> __device__ __forceinline__ void load_q(const AttentionPlan &p, const float *q, const Place &at, uint32_t h, f32x4 (&f)[DT]) {
    const uint32_t s = min(at.s0 + at.li, p.S - 1);
    const float *row = q + (((int64_t)at.b * p.S + s) * p.heads + h) * p.dim;
#pragma unroll
    for (int c = 0; c < DT; c++) {
        const uint32_t d = 16 * c + 4 * at.lg;
        f[c] = d < p.dim ? *reinterpret_cast<const f32x4 *>(row + d) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    }
}
template <int DT> __device__ __forceinline__ void load_k(const AttentionPlan &p, const Place &at, uint32_t g, uint32_t key, f32x4 (&f)[DT]) {
    const float *base = p.keys + ((int64_t)at.b * p.kv_heads + g) * p.k_block + (int64_t)key * p.dim; // (the same for the whole wave)
    const uint32_t row = min(at.li, p.cached + p.S - 1 - key) * p.dim + 4 * at.lg;
#pragma unroll
    for (int c = 0; c < DT; c++) {
        const uint32_t d = 16 * c + 4 * at.lg;
        f[c] = d < p.dim ? *reinterpret_cast<const f32x4 *>(base + (row + 16 * c)) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    }
}
// scores of 16 rows against 16 keys, before bias and mask
template <int DT> __device__ __forceinline__ f32x4 scores(const f32x4 (&q)[DT], const f32x4 (&k)[DT]) {
    f32x4 a = {0.0f, 0.0f, 0.0f, 0.0f}, b = a;
#pragma unroll
    for (int c = 0; c < DT; c += 2) { // two chains
#pragma unroll
        for (int t = 0; t < 4; t++) {
            a = mfma(q[c][t], k[c][t], a);
            if (c + 1 < DT) b = mfma(q[c + 1][t], k[c + 1][t], b);
        }
    }
    return a + b;
}
// whether every row of the tile sees every one of the 16 keys from j0
__device__ __forceinline__ bool all_visible(const AttentionPlan &p, uint32_t s0, uint32_t j0) {
    const uint32_t first = p.cached + s0, last = p.cached + min(s0 + kRowsT, p.S) - 1;
    return j0 + kKeysT - 1 <= first && (!p.window || last - j0 < p.window);
}
// A score with its distance bias; -inf when the row does not see the key, `d` (an exact integer) behind it.
__device__ __forceinline__ float biased(float v, float slope, bool whole, float d, float window) {
    v = fmaf(-slope, d, v);
    return whole || (d >= 0.0f && d < window) ? v : -INFINITY;
}
// Weights are 2^(score log2 e - top) times a scale per row, with `top` within kSlack of the row's largest score log2 e seen
// so far: close enough that nothing overflows, and it seldom has to move.
constexpr float kSlack = 24.0f;

template <int HPW, int DT>
__global__ __launch_bounds__(kStatWaves * 64) void attention_row_stats_kernel(const AttentionPlan p, const float *__restrict__ q, float2 *__restrict__ stats) {
    const uint32_t wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
    const Place at{blockIdx.z, tile_of(p, blockIdx.x, gridDim.x) * kRowsT, lane & 15, lane >> 4};
    const uint32_t h0 = (blockIdx.y * kStatWaves + wave) * HPW, rep = p.heads / p.kv_heads;
    if (h0 >= p.heads) return;
    f32x4 qf[HPW][DT];
    float slope[HPW], top[HPW][4], l[HPW][4];
    const float window = p.window ? (float)p.window : 3e38f, row = (float)(int)(p.cached + at.s0 + 4 * at.lg) - (float)at.li;
#pragma unroll
    for (int i = 0; i < HPW; i++) {
        const uint32_t h = min(h0 + i, p.heads - 1);
        load_q<DT>(p, q, at, h, qf[i]);
        slope[i] = p.bias ? slope_of(h, p.heads) : 0.0f;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            top[i][r] = p.zero_sink ? 0.0f : -1e30f; // (finite: a masked score against it weighs nothing)
            l[i][r] = 0.0f;
        }
    }
    uint32_t lo, hi;
    tile_keys(p, at.s0, &lo, &hi);
    const uint32_t g0 = h0 / rep;
    const bool shared = min(h0 + HPW - 1, p.heads - 1) / rep == g0; // one kv head for all of this wave's heads
    f32x4 next[DT];
    load_k<DT>(p, at, g0, lo, next);
    for (uint32_t j0 = lo; j0 < hi; j0 += kKeysT) {
        f32x4 k[DT];
#pragma unroll
        for (int c = 0; c < DT; c++) k[c] = next[c];
        if (j0 + kKeysT < hi) load_k<DT>(p, at, g0, j0 + kKeysT, next); // on its way while these are multiplied
        const bool whole = all_visible(p, at.s0, j0);
#pragma unroll
        for (int i = 0; i < HPW; i++) {
            if (i > 0 && !shared) load_k<DT>(p, at, min(h0 + i, p.heads - 1) / rep, j0, k);
            const f32x4 a = scores<DT>(qf[i], k);
            float x[4];
            bool moves = false;
#pragma unroll
            for (int r = 0; r < 4; r++) {
                x[r] = biased(a[r], slope[i], whole, row + (float)r - (float)j0, window);
                moves = moves || fmaf(x[r], kLog2e, -top[i][r]) > kSlack;
            }
            if (__any(moves)) {
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    float up = x[r] * kLog2e;
#pragma unroll
                    for (int d = 1; d < 16; d <<= 1) up = fmaxf(up, __shfl_xor(up, d, 64)); // over the lanes that share the row
                    up = fmaxf(top[i][r], up);
                    l[i][r] *= __builtin_amdgcn_exp2f(top[i][r] - up);
                    top[i][r] = up;
                }
            }
#pragma unroll
            for (int r = 0; r < 4; r++) l[i][r] += __builtin_amdgcn_exp2f(fmaf(x[r], kLog2e, -top[i][r]));
        }
    }
#pragma unroll
    for (int i = 0; i < HPW; i++) {
#pragma unroll
        for (int r = 0; r < 4; r++) {
            float sum = l[i][r];
#pragma unroll
            for (int d = 1; d < 16; d <<= 1) sum += __shfl_xor(sum, d, 64);
            if (p.zero_sink) sum += __builtin_amdgcn_exp2f(-top[i][r]);
            const uint32_t s = at.s0 + 4 * at.lg + r;
            if (at.li == 0 && s < p.S && h0 + i < p.heads) stats[((int64_t)at.b * p.S + s) * p.heads + h0 + i] = make_float2(top[i][r], 1.0f / sum);
        }
    }
}

// QREG: the queries stay in registers; else they are read again for every key tile.
template <int HPW, int DT, bool QREG, bool TALK>
__global__ __launch_bounds__(kTileWaves * 64) void attention_tiles_kernel(const AttentionPlan p, const float *__restrict__ q, const float2 *__restrict__ stats,
                                                                          const uint32_t tiles, const uint32_t splits, float *__restrict__ dst) {
    extern __shared__ float lds[]; // three buffers of weights [heads rounded up to 16][16][16]
    constexpr int RT = (HPW * kTileWaves + 15) / 16; // row tiles of the mixing product
    const uint32_t wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
    const uint32_t tile = tile_of(p, blockIdx.x / splits, tiles), split = blockIdx.x % splits;
    const Place at{blockIdx.y, tile * kRowsT, lane & 15, lane >> 4};
    const uint32_t h0 = wave * HPW, rep = p.heads / p.kv_heads, tiles16 = (p.heads + 15) / 16, buffer = tiles16 * 16 * kHeadPitch;
    const bool shared = min(h0 + HPW - 1, p.heads - 1) / rep == min(h0, p.heads - 1) / rep; // one kv head for all of this wave's heads
    uint32_t lo, hi;
    tile_keys(p, at.s0, &lo, &hi);
    // this workgroup's part of the keys, in whole key tiles
    const uint32_t ntiles = (hi - lo + kKeysT - 1) / kKeysT, per = (ntiles + splits - 1) / splits;
    const uint32_t first = min(ntiles, split * per), n = min(ntiles, first + per) - first;
    lo += first * kKeysT;
    const float window = p.window ? (float)p.window : 3e38f, row = (float)(int)(p.cached + at.s0 + 4 * at.lg) - (float)at.li;

    f32x4 qf[QREG ? HPW : 1][DT], out[HPW][DT];
    float slope[HPW];
    // the rows' maxima and scales [heads][16] each, and talk [heads rounded up][the same + 4], behind the buffers
    const uint32_t talk_pitch = tiles16 * 16 + 4;
    float *tops = lds + 3 * buffer, *scales = tops + p.heads * kRowsT, *talk = scales + p.heads * kRowsT;
#pragma unroll
    for (int i = 0; i < HPW; i++) {
        const uint32_t h = min(h0 + i, p.heads - 1);
        if constexpr (QREG) load_q<DT>(p, q, at, h, qf[i]);
        slope[i] = p.bias ? slope_of(h, p.heads) : 0.0f;
#pragma unroll
        for (int c = 0; c < DT; c++) out[i][c] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    }
    for (uint32_t i = threadIdx.x; i < p.heads * kRowsT; i += kTileWaves * 64) {
        const float2 st = stats[((int64_t)at.b * p.S + min(at.s0 + i % kRowsT, p.S - 1)) * p.heads + i / kRowsT];
        tops[i] = st.x;
        scales[i] = st.y;
    }
    if constexpr (TALK) {
        for (uint32_t i = threadIdx.x; i < tiles16 * 16 * tiles16 * 16; i += kTileWaves * 64) {
            const uint32_t h = i / (tiles16 * 16), g = i % (tiles16 * 16);
            talk[h * talk_pitch + g] = h < p.heads && g < p.heads ? p.talk[(int64_t)h * p.heads + g] : 0.0f;
        }
        for (uint32_t i = p.heads * kHeadPitch + threadIdx.x; i < buffer; i += kTileWaves * 64) // heads that are not there
            lds[i] = lds[buffer + i] = lds[2 * buffer + i] = 0.0f;
    }
    __syncthreads();
    constexpr uint32_t LAG = TALK ? 1 : 0; // tiles that the mixing runs behind the scores, and the values behind the mixing
    uint32_t b0 = 0, b1 = 2, b2 = 1;       // buffers of this iteration's scores, mixing, values
    for (uint32_t it = 0; it < n + 2 * LAG; it++) {
        const bool do_s = it < n && h0 < p.heads, do_v = it >= 2 * LAG && h0 < p.heads;
        const uint32_t js = lo + it * kKeysT, jv = lo + (it - 2 * LAG) * kKeysT, last = p.cached + p.S - 1;
        f32x4 k[DT];
        float v[4][DT];
        auto load_v = [&](uint32_t g) {
            const float *base = p.values + ((int64_t)at.b * p.kv_heads + g) * p.v_block + (int64_t)jv * p.vdim;
#pragma unroll
            for (int t = 0; t < 4; t++) {
                const uint32_t row = min(4 * at.lg + t, last - jv) * p.vdim + at.li;
#pragma unroll
                for (int c = 0; c < DT; c++) v[t][c] = 16 * c + at.li < p.vdim ? base[row + 16 * c] : 0.0f;
            }
        };
        if (do_s) load_k<DT>(p, at, h0 / rep, js, k);
        if (do_v && LAG) load_v(h0 / rep);
        if (TALK && it >= LAG && it < n + LAG) {
            // talk [heads, heads] . weights [heads, 256 columns]: a wave owns whole columns and writes them back in place
#pragma unroll
            for (uint32_t e = 0; e < kRowsT / kTileWaves; e++) {
                float *w = lds + b1 * buffer + (wave * (kRowsT / kTileWaves) + e) * kRowPitch + at.li;
                f32x4 acc[RT];
#pragma unroll
                for (int a = 0; a < RT; a++) acc[a] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
                for (int c = 0; c < RT; c++) {
                    if (c >= (int)tiles16) break;
                    f32x4 f[RT];
#pragma unroll
                    for (int a = 0; a < RT; a++)
                        f[a] = *reinterpret_cast<const f32x4 *>(talk + min(16 * a + at.li, tiles16 * 16 - 1) * talk_pitch + 16 * c + 4 * at.lg);
#pragma unroll
                    for (int t = 0; t < 4; t++) {
                        const float x = w[(16 * c + 4 * at.lg + t) * kHeadPitch];
#pragma unroll
                        for (int a = 0; a < RT; a++) acc[a] = mfma(f[a][t], x, acc[a]);
                    }
                }
#pragma unroll
                for (int a = 0; a < RT; a++)
#pragma unroll
                    for (int r = 0; r < 4; r++) {
                        const uint32_t h = 16 * a + 4 * at.lg + r;
                        if (h < p.heads) w[h * kHeadPitch] = acc[a][r];
                    }
            }
        }
        if (do_s) { // scores -> weights of this wave's heads
            const bool whole = all_visible(p, at.s0, js);
#pragma unroll
            for (int i = 0; i < HPW; i++) {
                const uint32_t h = h0 + i;
                if (h >= p.heads) break;
                if (i > 0 && !shared) load_k<DT>(p, at, h / rep, js, k);
                if constexpr (!QREG) load_q<DT>(p, q, at, h, qf[0]);
                const f32x4 a = scores<DT>(qf[QREG ? i : 0], k);
                float *w = lds + b0 * buffer + h * kHeadPitch + at.li;
                const f32x4 top = *reinterpret_cast<const f32x4 *>(tops + h * kRowsT + 4 * at.lg), scale = *reinterpret_cast<const f32x4 *>(scales + h * kRowsT + 4 * at.lg);
#pragma unroll
                for (int r = 0; r < 4; r++)
                    w[(4 * at.lg + r) * kRowPitch] =
                        __builtin_amdgcn_exp2f(fmaf(biased(a[r], slope[i], whole, row + (float)r - (float)js, window), kLog2e, -top[r])) * scale[r];
            }
        }
        if (do_v) { // weights . values
#pragma unroll
            for (int i = 0; i < HPW; i++) {
                const uint32_t h = h0 + i;
                if (h >= p.heads) break;
                if ((i == 0 && !LAG) || (i > 0 && !shared)) load_v(h / rep);
                const f32x4 w = *reinterpret_cast<const f32x4 *>(lds + (LAG ? b2 : b0) * buffer + h * kHeadPitch + at.li * kRowPitch + 4 * at.lg);
#pragma unroll
                for (int t = 0; t < 4; t++)
#pragma unroll
                    for (int c = 0; c < DT; c++) out[i][c] = mfma(w[t], v[t][c], out[i][c]);
            }
        }
        if constexpr (TALK) __syncthreads();
        const uint32_t b = b2;
        b2 = b1;
        b1 = b0;
        b0 = b;
    }
    float *o = dst + (int64_t)split * p.B * p.S * p.heads * p.vdim;
#pragma unroll
    for (int i = 0; i < HPW; i++) {
        const uint32_t h = h0 + i;
        if (h >= p.heads) break;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const uint32_t s = at.s0 + 4 * at.lg + r;
            if (s >= p.S) continue;
            float *row = o + (((int64_t)at.b * p.S + s) * p.heads + h) * p.vdim + at.li;
#pragma unroll
            for (int c = 0; c < DT; c++)
                if (16 * c + at.li < p.vdim) row[16 * c] = out[i][c][r];
        }
    }
}

// out = the parts added up
__global__ __launch_bounds__(256) void attention_parts_kernel(const float *__restrict__ parts, const uint32_t splits, const uint64_t n, float *__restrict__ out) {
    const uint64_t i = ((uint64_t)blockIdx.x * 256 + threadIdx.x) * 4;
    if (i >= n) return;
    if (i + 4 <= n && n % 4 == 0) {
        f32x4 s = *reinterpret_cast<const f32x4 *>(parts + i);
        for (uint32_t k = 1; k < splits; k++) s += *reinterpret_cast<const f32x4 *>(parts + k * n + i);
        *reinterpret_cast<f32x4 *>(out + i) = s;
    } else {
        for (uint64_t e = i; e < min(i + 4, n); e++) {
            float s = parts[e];
            for (uint32_t k = 1; k < splits; k++) s += parts[k * n + e];
            out[e] = s;
        }
    }
}

template <int HPW, int DT, bool QREG> int run_tiles(cg_backend *be, const AttentionPlan &p, const float *q, float2 *stats, uint32_t splits, float *dst) {
    const uint32_t tiles = (p.S + kRowsT - 1) / kRowsT, rep = p.heads / p.kv_heads;
    // heads of a stats wave: two that share their keys, or one
    if (rep % 2 == 0 && DT <= 4)
        hipLaunchKernelGGL((attention_row_stats_kernel<2, DT>), dim3(tiles, (p.heads + 2 * kStatWaves - 1) / (2 * kStatWaves), p.B), dim3(kStatWaves * 64), 0,
                           be->stream, p, q, stats);
    else
        hipLaunchKernelGGL((attention_row_stats_kernel<1, DT>), dim3(tiles, (p.heads + kStatWaves - 1) / kStatWaves, p.B), dim3(kStatWaves * 64), 0, be->stream, p,
                           q, stats);
    const size_t h16 = (p.heads + 15) / 16 * 16, lds = (3 * h16 * kHeadPitch + 2 * p.heads * kRowsT + h16 * (h16 + 4)) * 4;
    const void *f = p.talk ? reinterpret_cast<const void *>(&attention_tiles_kernel<HPW, DT, QREG, true>)
                           : reinterpret_cast<const void *>(&attention_tiles_kernel<HPW, DT, QREG, false>);
    if (lds > (64 << 10)) {
        const hipError_t e = hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return hip_fail(e, "hipFuncSetAttribute");
    }
    const dim3 grid(tiles * splits, p.B);
    if (p.talk) hipLaunchKernelGGL((attention_tiles_kernel<HPW, DT, QREG, true>), grid, dim3(kTileWaves * 64), lds, be->stream, p, q, stats, tiles, splits, dst);
    else hipLaunchKernelGGL((attention_tiles_kernel<HPW, DT, QREG, false>), grid, dim3(kTileWaves * 64), lds, be->stream, p, q, stats, tiles, splits, dst);
    return CG_OK;
}
template <int HPW> int run_tiles(cg_backend *be, const AttentionPlan &p, const float *q, float2 *stats, uint32_t splits, float *dst) {
    const uint32_t d = std::max(p.dim, p.vdim);
    if (d <= 32) return run_tiles<HPW, 2, true>(be, p, q, stats, splits, dst);
    if (d <= 64) return run_tiles<HPW, 4, true>(be, p, q, stats, splits, dst);
    if (d <= 96) return run_tiles<HPW, 6, (HPW < 4)>(be, p, q, stats, splits, dst);
    return run_tiles<HPW, 8, (HPW < 4)>(be, p, q, stats, splits, dst);
}

} // namespace

int launch_attention_tiles(cg_backend *be, const AttentionPlan &p, const float *q) {
    if (p.S <= kFewRows || p.heads > 32 || p.dim % 4 || p.dim > 128 || p.vdim > 128 || p.B > 65535) return kDeclined;
    const uint64_t n = (uint64_t)p.B * p.S * p.heads * p.vdim;
    const uint32_t tiles = (p.S + kRowsT - 1) / kRowsT, keys = p.cached + p.S, most = p.window ? std::min(p.window + kRowsT, keys) : keys;
    // too few row tiles for the device: their keys are cut over up to 4 workgroups, each with at least 8 key tiles
    const uint32_t want = (uint32_t)(2 * be->compute_units) / std::max(1u, tiles * p.B);
    const uint32_t splits = std::max(1u, std::min(std::min(4u, want), most / (8 * kKeysT)));
    void *mem = nullptr, *parts = nullptr;
    size_t mem_cls = 0, parts_cls = 0;
    int rc = be->pool.alloc((size_t)p.B * p.S * p.heads * sizeof(float2), &mem, &mem_cls);
    if (!rc && splits > 1) rc = be->pool.alloc((size_t)n * splits * 4, &parts, &parts_cls);
    float *dst = splits > 1 ? static_cast<float *>(parts) : p.out;
    float2 *stats = static_cast<float2 *>(mem);
    if (!rc)
        rc = p.heads <= 8    ? run_tiles<1>(be, p, q, stats, splits, dst)
             : p.heads <= 16 ? run_tiles<2>(be, p, q, stats, splits, dst)
                             : run_tiles<4>(be, p, q, stats, splits, dst);
    if (!rc && splits > 1)
        hipLaunchKernelGGL(attention_parts_kernel, dim3((uint32_t)((n + 1023) / 1024)), dim3(256), 0, be->stream, dst, splits, n, p.out);
    if (mem) be->pool.free(mem, mem_cls);
    if (parts) be->pool.free(parts, parts_cls);
    if (rc) return rc;
    const hipError_t e = hipGetLastError();
    return e == hipSuccess ? CG_OK : hip_fail(e, "block_attention");
}

} // namespace cg
