// cg_block_attention for more than a few new tokens: 16 query rows of all heads against 32 keys at a time, every product on
// v_mfma_f32_16x16x4.  Head mixing after the soft-max needs the finished weights of every head for the same (query, key),
// so the row maxima and sums come first, from a launch of their own:
//
//   attention_row_stats_kernel  a wave per (16 query rows, one or two heads): maximum and sum of every row's scores
//   attention_tiles_kernel      8 or 16 waves per 16 query rows, one or two heads each: scores again, weights to LDS, mixed there over
//                               the heads (as the product talk . weights, a column per (query, key)), times the values.
//                               The keys of a row tile may be cut over several workgroups: finished weights only add up.
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

constexpr int kStatWaves = 4;
constexpr uint32_t kRowsT = 16, kKeysT = 32;
constexpr uint32_t kRowPitch = kKeysT + 4;                // floats; 16-byte rows off each other's banks
constexpr uint32_t kHeadPitch = kRowsT * kRowPitch + 4;   // heads four apart lie 16 banks apart
constexpr float kLog2e = 1.44269504088896341f;

__device__ __forceinline__ float exp_of(float x) { return __builtin_amdgcn_exp2f(x * kLog2e); } // (x <= 0)
__device__ __forceinline__ f32x4 mfma(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
__device__ __forceinline__ float slope_of(uint32_t h, uint32_t heads) { return exp2f(-8.0f * (float)(h + 1) / (float)heads); }

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
    const float *row = p.keys + ((int64_t)at.b * p.kv_heads + g) * p.k_block + (int64_t)min(key + at.li, p.cached + p.S - 1) * p.dim;
#pragma unroll
    for (int c = 0; c < DT; c++) {
        const uint32_t d = 16 * c + 4 * at.lg;
        f[c] = d < p.dim ? *reinterpret_cast<const f32x4 *>(row + d) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
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
// score of row s (register r) and key j with bias; -inf when the row does not see the key
__device__ __forceinline__ float visible_score(const AttentionPlan &p, float v, float slope, uint32_t s, uint32_t j, uint32_t end) {
    const int d = (int)(p.cached + s) - (int)j;
    v -= slope * (float)d;
    return d >= 0 && (!p.window || d < (int)p.window) && j < end ? v : -INFINITY;
}

template <int HPW, int DT>
__global__ __launch_bounds__(kStatWaves * 64) void attention_row_stats_kernel(const AttentionPlan p, const float *__restrict__ q, float2 *__restrict__ stats) {
    const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const Place at{blockIdx.z, blockIdx.x * kRowsT, lane & 15, lane >> 4};
    const uint32_t h0 = (blockIdx.y * kStatWaves + wave) * HPW, rep = p.heads / p.kv_heads;
    if (h0 >= p.heads) return;
    f32x4 qf[HPW][DT];
    float slope[HPW], m[HPW][4], l[HPW][4];
#pragma unroll
    for (int i = 0; i < HPW; i++) {
        const uint32_t h = min(h0 + i, p.heads - 1);
        load_q<DT>(p, q, at, h, qf[i]);
        slope[i] = p.bias ? slope_of(h, p.heads) : 0.0f;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            m[i][r] = -1e30f; // (finite: a masked score against it weighs nothing)
            l[i][r] = 0.0f;
        }
    }
    uint32_t lo, hi;
    tile_keys(p, at.s0, &lo, &hi);
    const uint32_t g0 = h0 / rep;
    const bool shared = min(h0 + HPW - 1, p.heads - 1) / rep == g0; // one kv head for all of this wave's heads
    for (uint32_t j0 = lo; j0 < hi; j0 += 16) {
        f32x4 k[DT];
        load_k<DT>(p, at, g0, j0, k);
#pragma unroll
        for (int i = 0; i < HPW; i++) {
            if (i > 0 && !shared) load_k<DT>(p, at, min(h0 + i, p.heads - 1) / rep, j0, k);
            const f32x4 a = scores<DT>(qf[i], k);
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const float x = visible_score(p, a[r], slope[i], at.s0 + 4 * at.lg + r, j0 + at.li, hi);
                const float up = fmaxf(m[i][r], x);
                // one of the two factors is 1
                const float e = exp_of(fminf(m[i][r], x) - up);
                l[i][r] = x > m[i][r] ? fmaf(l[i][r], e, 1.0f) : l[i][r] + e;
                m[i][r] = up;
            }
        }
    }
#pragma unroll
    for (int i = 0; i < HPW; i++) {
#pragma unroll
        for (int r = 0; r < 4; r++) {
            float top = m[i][r];
#pragma unroll
            for (int d = 1; d < 16; d <<= 1) top = fmaxf(top, __shfl_xor(top, d, 64));
            float sum = l[i][r] * exp_of(m[i][r] - top);
#pragma unroll
            for (int d = 1; d < 16; d <<= 1) sum += __shfl_xor(sum, d, 64);
            const uint32_t s = at.s0 + 4 * at.lg + r;
            if (at.li == 0 && s < p.S && h0 + i < p.heads) stats[((int64_t)at.b * p.S + s) * p.heads + h0 + i] = make_float2(top, 1.0f / sum);
        }
    }
}

// QREG: the queries stay in registers; else they are read again for every key tile.
template <int NW, int HPW, int DT, bool QREG, bool TALK>
__global__ __launch_bounds__(NW * 64) void attention_tiles_kernel(const AttentionPlan p, const float *__restrict__ q, const float2 *__restrict__ stats,
                                                                          const uint32_t splits, float *__restrict__ dst) {
    extern __shared__ float lds[]; // weights [heads rounded up to 16][16][32]
    constexpr int RT = (HPW * NW + 15) / 16; // row tiles of the mixing product
    const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const uint32_t tile = blockIdx.x / splits, split = blockIdx.x - tile * splits;
    const Place at{blockIdx.y, tile * kRowsT, lane & 15, lane >> 4};
    const uint32_t h0 = wave * HPW, rep = p.heads / p.kv_heads, tiles16 = (p.heads + 15) / 16;
    uint32_t lo, hi;
    tile_keys(p, at.s0, &lo, &hi);
    // this workgroup's part of the keys, in whole key tiles
    const uint32_t ntiles = (hi - lo + kKeysT - 1) / kKeysT, per = (ntiles + splits - 1) / splits;
    const uint32_t end = hi;
    hi = min(hi, lo + (split + 1) * per * kKeysT);
    lo += split * per * kKeysT;

    const bool shared = min(h0 + HPW - 1, p.heads - 1) / rep == min(h0, p.heads - 1) / rep; // one kv head for all of this wave's heads

    f32x4 qf[QREG ? HPW : 1][DT], out[HPW][DT], talk[TALK ? RT : 1][TALK ? RT : 1];
    float slope[HPW], top[HPW][4], scale[HPW][4];
#pragma unroll
    for (int i = 0; i < HPW; i++) {
        const uint32_t h = min(h0 + i, p.heads - 1);
        if constexpr (QREG) load_q<DT>(p, q, at, h, qf[i]);
        slope[i] = p.bias ? slope_of(h, p.heads) : 0.0f;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const float2 st = stats[((int64_t)at.b * p.S + min(at.s0 + 4 * at.lg + r, p.S - 1)) * p.heads + h];
            top[i][r] = st.x;
            scale[i][r] = st.y;
        }
#pragma unroll
        for (int c = 0; c < DT; c++) out[i][c] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    }
    if constexpr (TALK) {
#pragma unroll
        for (int a = 0; a < RT; a++)
#pragma unroll
            for (int c = 0; c < RT; c++)
#pragma unroll
                for (int t = 0; t < 4; t++) {
                    const uint32_t h = 16 * a + at.li, g = 16 * c + 4 * at.lg + t;
                    talk[a][c][t] = h < p.heads && g < p.heads ? p.talk[(int64_t)h * p.heads + g] : 0.0f;
                }
        for (uint32_t i = p.heads * kHeadPitch + threadIdx.x; i < tiles16 * 16 * kHeadPitch; i += NW * 64) lds[i] = 0.0f; // heads that are not there
    }
    for (uint32_t j0 = lo; j0 < hi; j0 += kKeysT) {
        // scores -> weights of this wave's heads
#pragma unroll
        for (int half = 0; half < 2; half++) {
            f32x4 k[DT];
            if (h0 < p.heads) load_k<DT>(p, at, h0 / rep, j0 + 16 * half, k);
#pragma unroll
            for (int i = 0; i < HPW; i++) {
                const uint32_t h = h0 + i;
                if (h >= p.heads) break;
                if (i > 0 && !shared) load_k<DT>(p, at, h / rep, j0 + 16 * half, k);
                if constexpr (!QREG) load_q<DT>(p, q, at, h, qf[0]);
                const f32x4 a = scores<DT>(qf[QREG ? i : 0], k);
                float *w = lds + h * kHeadPitch + 16 * half + at.li;
#pragma unroll
                for (int r = 0; r < 4; r++)
                    w[(4 * at.lg + r) * kRowPitch] =
                        exp_of(visible_score(p, a[r], slope[i], at.s0 + 4 * at.lg + r, j0 + 16 * half + at.li, end) - top[i][r]) * scale[i][r];
            }
        }
        if constexpr (TALK) {
            __syncthreads();
            // talk [heads, heads] . weights [heads, 512 columns]: a wave owns whole columns and writes them back in place
#pragma unroll
            for (uint32_t n = 0; n < kRowsT * kKeysT / 16 / NW; n++) {
                const uint32_t col = (wave * (kRowsT * kKeysT / 16 / NW) + n) * 16; // of 512
                float *w = lds + (col / kKeysT) * kRowPitch + (col % kKeysT) + at.li;
                f32x4 acc[RT];
#pragma unroll
                for (int a = 0; a < RT; a++) acc[a] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
                for (int c = 0; c < RT; c++) {
                    if (c >= (int)tiles16) break;
#pragma unroll
                    for (int t = 0; t < 4; t++) {
                        const float v = w[(16 * c + 4 * at.lg + t) * kHeadPitch];
#pragma unroll
                        for (int a = 0; a < RT; a++) acc[a] = mfma(talk[a][c][t], v, acc[a]);
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
            __syncthreads();
        }
        // weights . values
#pragma unroll
        for (int half = 0; half < 2; half++) {
            float v[4][DT];
#pragma unroll
            for (int i = 0; i < HPW; i++) {
                const uint32_t h = h0 + i;
                if (h >= p.heads) break;
                const uint32_t g = h / rep;
                if (i == 0 || !shared) {
#pragma unroll
                    for (int t = 0; t < 4; t++) {
                        const float *row = p.values + ((int64_t)at.b * p.kv_heads + g) * p.v_block +
                                           (int64_t)min(j0 + 16 * half + 4 * at.lg + t, p.cached + p.S - 1) * p.vdim + at.li;
#pragma unroll
                        for (int c = 0; c < DT; c++) v[t][c] = 16 * c + at.li < p.vdim ? row[16 * c] : 0.0f;
                    }
                }
                const f32x4 w = *reinterpret_cast<const f32x4 *>(lds + h * kHeadPitch + at.li * kRowPitch + 16 * half + 4 * at.lg);
#pragma unroll
                for (int t = 0; t < 4; t++)
#pragma unroll
                    for (int c = 0; c < DT; c++) out[i][c] = mfma(w[t], v[t][c], out[i][c]);
            }
        }
        if constexpr (TALK) __syncthreads(); // the next weights overwrite these
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

template <int NW, int HPW, int DT, bool QREG> int run_tiles(cg_backend *be, const AttentionPlan &p, const float *q, float2 *stats, uint32_t splits, float *dst) {
    const uint32_t tiles = (p.S + kRowsT - 1) / kRowsT, rep = p.heads / p.kv_heads;
    // heads of a stats wave: two that share their keys, or one
    if (rep % 2 == 0 && DT <= 4)
        hipLaunchKernelGGL((attention_row_stats_kernel<2, DT>), dim3(tiles, (p.heads + 2 * kStatWaves - 1) / (2 * kStatWaves), p.B), dim3(kStatWaves * 64), 0,
                           be->stream, p, q, stats);
    else
        hipLaunchKernelGGL((attention_row_stats_kernel<1, DT>), dim3(tiles, (p.heads + kStatWaves - 1) / kStatWaves, p.B), dim3(kStatWaves * 64), 0, be->stream, p,
                           q, stats);
    const size_t lds = (size_t)(p.heads + 15) / 16 * 16 * kHeadPitch * 4;
    const void *f = p.talk ? reinterpret_cast<const void *>(&attention_tiles_kernel<NW, HPW, DT, QREG, true>)
                           : reinterpret_cast<const void *>(&attention_tiles_kernel<NW, HPW, DT, QREG, false>);
    if (lds > (64 << 10)) {
        const hipError_t e = hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return hip_fail(e, "hipFuncSetAttribute");
    }
    const dim3 grid(tiles * splits, p.B);
    if (p.talk) hipLaunchKernelGGL((attention_tiles_kernel<NW, HPW, DT, QREG, true>), grid, dim3(NW * 64), lds, be->stream, p, q, stats, splits, dst);
    else hipLaunchKernelGGL((attention_tiles_kernel<NW, HPW, DT, QREG, false>), grid, dim3(NW * 64), lds, be->stream, p, q, stats, splits, dst);
    return CG_OK;
}
template <int NW, int HPW> int run_tiles(cg_backend *be, const AttentionPlan &p, const float *q, float2 *stats, uint32_t splits, float *dst) {
    const uint32_t d = std::max(p.dim, p.vdim);
    if (d <= 32) return run_tiles<NW, HPW, 2, true>(be, p, q, stats, splits, dst);
    if (d <= 64) return run_tiles<NW, HPW, 4, true>(be, p, q, stats, splits, dst);
    if (d <= 96) return run_tiles<NW, HPW, 6, (HPW < 2)>(be, p, q, stats, splits, dst);
    return run_tiles<NW, HPW, 8, (HPW < 2)>(be, p, q, stats, splits, dst);
}

} // namespace

int launch_attention_tiles(cg_backend *be, const AttentionPlan &p, const float *q) {
    if (p.S <= kFewRows || p.heads > 32 || p.dim % 4 || p.dim > 128 || p.vdim > 128 || p.B > 65535) return kDeclined;
    const uint64_t n = (uint64_t)p.B * p.S * p.heads * p.vdim;
    const uint32_t tiles = (p.S + kRowsT - 1) / kRowsT, keys = p.cached + p.S, most = p.window ? std::min(p.window + kRowsT, keys) : keys;
    // too few row tiles for the device: their keys are cut over up to 4 workgroups, each with at least 4 key tiles
    const uint32_t want = (uint32_t)(2 * be->compute_units) / std::max(1u, tiles * p.B);
    const uint32_t splits = std::max(1u, std::min(std::min(4u, want), most / (4 * kKeysT)));
    void *mem = nullptr, *parts = nullptr;
    size_t mem_cls = 0, parts_cls = 0;
    int rc = be->pool.alloc((size_t)p.B * p.S * p.heads * sizeof(float2), &mem, &mem_cls);
    if (!rc && splits > 1) rc = be->pool.alloc((size_t)n * splits * 4, &parts, &parts_cls);
    float *dst = splits > 1 ? static_cast<float *>(parts) : p.out;
    float2 *stats = static_cast<float2 *>(mem);
    if (!rc)
        rc = p.heads <= 8    ? run_tiles<8, 1>(be, p, q, stats, splits, dst)
             : p.heads <= 16 ? run_tiles<16, 1>(be, p, q, stats, splits, dst)
                             : run_tiles<16, 2>(be, p, q, stats, splits, dst);
    if (!rc && splits > 1)
        hipLaunchKernelGGL(attention_parts_kernel, dim3((uint32_t)((n + 1023) / 1024)), dim3(256), 0, be->stream, dst, splits, n, p.out);
    if (mem) be->pool.free(mem, mem_cls);
    if (parts) be->pool.free(parts, parts_cls);
    if (rc) return rc;
    const hipError_t e = hipGetLastError();
    return e == hipSuccess ? CG_OK : hip_fail(e, "block_attention");
}

} // namespace cg
