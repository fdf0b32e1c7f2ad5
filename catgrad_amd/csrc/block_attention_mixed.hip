// cg_block_attention when the scores are mixed over the heads before the soft-max.  A query's mixed scores need every head's
// score for the same key, but no other key's: the soft-max runs along, its results unfinished until the largest score and the
// sum are known.
//
//   attention_mixed_step_kernel   a few new tokens: a workgroup per (token, segment of keys) for all heads, from the projections
//                                 as they are to the segment's weighted values
//   attention_mixed_tiles_kernel  prompts: 16 query rows of all heads against 16 keys at a time on v_mfma_f32_16x16x4; scores,
//                                 mixing (the product talk . scores, a column per (query, key)) and soft-max with values run a
//                                 key tile apart on three buffers, one barrier per tile
//   attention_mixed_rows_kernel   other sizes: behind attention_scores_kernel, a workgroup per (token, kv head, 128 keys)
//   attention_merge_kernel        the segments' unfinished results, each with its largest score and sum, become one
//
// Unfinished results carry {top, sum}: weights are 2^(score log2 e - top), `top` in units of log2.
#include "blocks.hpp"
#include "device_utils.hpp"

#include <algorithm>
#include <type_traits>

namespace cg {
namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));
constexpr int kThreads = 256;
constexpr uint32_t kSeg = 128; // keys of a segment of attention_scores_kernel
constexpr float kLog2e = 1.44269504088896341f, kNone = -1e30f;

__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
    for (int d = 32; d > 0; d >>= 1) v = fmaxf(v, __shfl_xor(v, d, 64));
    return v;
}
__device__ __forceinline__ float slope_of(uint32_t h, uint32_t heads) { return exp2f(-8.0f * (float)(h + 1) / (float)heads); }
__device__ __forceinline__ uint32_t first_visible(const AttentionPlan &p, uint32_t i) { return p.window && i + 1 > p.window ? i + 1 - p.window : 0; }

// out = the segments' results together; result i of a row: head i / vdim.  parts at row * row_pitch + segment * seg_pitch,
// stats the same in heads.  A workgroup per 64 results, its waves a run of segments each.
constexpr int kMergeWaves = 8;
__global__ __launch_bounds__(kMergeWaves * 64) void attention_merge_kernel(const float *__restrict__ parts, const float2 *__restrict__ stats, const uint32_t segs,
                                                                           const uint64_t row_pitch, const uint64_t seg_pitch, const uint32_t heads, const uint32_t vdim,
                                                                           const bool sink, float *__restrict__ out) {
    __shared__ float sums[3][kMergeWaves][64];
    const uint32_t n = heads * vdim, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, i = min(blockIdx.x * 64 + lane, n - 1);
    const uint64_t row = blockIdx.y;
    const float *p = parts + row * row_pitch * vdim + i;
    const float2 *st = stats + row * row_pitch + i / vdim;
    const uint32_t per = (segs + kMergeWaves - 1) / kMergeWaves, k0 = min(segs, wave * per), k1 = min(segs, k0 + per);
    float m = kNone, l = 0.0f, o = 0.0f;
    constexpr int AHEAD = 8;
    for (uint32_t k = k0; k < k1; k += AHEAD) {
        float2 t[AHEAD];
        float v[AHEAD];
#pragma unroll
        for (int e = 0; e < AHEAD; e++) { // (clamped: a segment behind the last weighs nothing)
            const uint64_t at = (uint64_t)min(k + e, k1 - 1) * seg_pitch;
            t[e] = st[at];
            v[e] = p[at * vdim];
            if (k + e >= k1) t[e] = make_float2(kNone, 0.0f);
        }
        float up = m;
#pragma unroll
        for (int e = 0; e < AHEAD; e++) up = fmaxf(up, t[e].x);
        const float f = __builtin_amdgcn_exp2f(m - up);
        l *= f;
        o *= f;
        m = up;
#pragma unroll
        for (int e = 0; e < AHEAD; e++) {
            const float w = k + e < k1 ? __builtin_amdgcn_exp2f(t[e].x - m) : 0.0f;
            l = fmaf(t[e].y, w, l);
            o = fmaf(v[e], w, o);
        }
    }
    sums[0][wave][lane] = m;
    sums[1][wave][lane] = l;
    sums[2][wave][lane] = o;
    __syncthreads();
    if (wave) return;
    m = sink ? 0.0f : kNone;
#pragma unroll
    for (int w = 0; w < kMergeWaves; w++) m = fmaxf(m, sums[0][w][lane]);
    l = sink ? __builtin_amdgcn_exp2f(-m) : 0.0f;
    o = 0.0f;
#pragma unroll
    for (int w = 0; w < kMergeWaves; w++) {
        const float f = __builtin_amdgcn_exp2f(sums[0][w][lane] - m);
        l = fmaf(sums[1][w][lane], f, l);
        o = fmaf(sums[2][w][lane], f, o);
    }
    if (blockIdx.x * 64 + lane < n) out[row * n + i] = o / l;
}

// ---- other sizes -----------------------------------------------------------------------------------------------------
__host__ __device__ constexpr uint32_t mixed_floats(uint32_t rep, uint32_t slots, uint32_t vw) { return slots * kSeg + rep * kSeg + rep * vw * kThreads; }

template <int REP, int VW>
__global__ __launch_bounds__(kThreads) void attention_mixed_rows_kernel(const AttentionPlan p, const uint32_t row0, const uint32_t nseg, const float *__restrict__ scores,
                                                                        float *__restrict__ parts, float2 *__restrict__ stats) {
    extern __shared__ float lds[];
    const uint32_t rep = p.heads / p.kv_heads, groups = (rep + REP - 1) / REP;
    const uint32_t g = blockIdx.y / groups, h0 = g * rep + (blockIdx.y - g * groups) * REP, nh = min((uint32_t)REP, (g + 1) * rep - h0);
    const uint32_t r = row0 + blockIdx.z, b = r / p.S, s = r - b * p.S, seg = blockIdx.x;
    const uint32_t first = p.talk ? 0 : h0, nm = p.talk ? p.heads : nh, slots = p.talk ? p.heads : REP;
    float *raw = lds, *wt = raw + slots * kSeg, *red = wt + REP * kSeg;
    const uint32_t hi = p.cached + s + 1, j0 = first_visible(p, p.cached + s) + seg * kSeg, keys = j0 < hi ? min(kSeg, hi - j0) : 0;
    const uint32_t key = threadIdx.x % kSeg; // two threads share a key's column of scores
    for (uint32_t h = threadIdx.x / kSeg; h < nm; h += kThreads / kSeg)
        raw[h * kSeg + key] = key < keys ? scores[(((int64_t)blockIdx.z * p.heads + first + h) * nseg + seg) * kSeg + key] : 0.0f;
    __syncthreads();
    for (uint32_t o = threadIdx.x / kSeg; o < nh; o += kThreads / kSeg) {
        float w = 0.0f;
        if (p.talk) {
            for (uint32_t h = 0; h < nm; h++) w = fmaf(p.talk[(int64_t)(h0 + o) * p.heads + h], raw[h * kSeg + key], w);
        } else {
            w = raw[o * kSeg + key];
        }
        wt[o * kSeg + key] = key < keys ? w * kLog2e : -INFINITY;
    }
    __syncthreads();
    const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    for (uint32_t o = wave; o < nh; o += kThreads / 64) {
        const float a = wt[o * kSeg + lane], c = wt[o * kSeg + 64 + lane];
        const float m = fmaxf(kNone, wave_max(fmaxf(a, c)));
        const float ea = __builtin_amdgcn_exp2f(a - m), ec = __builtin_amdgcn_exp2f(c - m), l = wave_total(ea + ec);
        wt[o * kSeg + lane] = ea;
        wt[o * kSeg + 64 + lane] = ec;
        if (lane == 0) stats[((int64_t)blockIdx.z * nseg + seg) * p.heads + h0 + o] = make_float2(m, l);
    }
    __syncthreads();
    const float *V = p.values + ((int64_t)b * p.kv_heads + g) * p.v_block + (int64_t)min(j0, hi - 1) * p.vdim;
    uint32_t lanes = 1; // lanes side by side along vdim; the others take keys in turn
    while (lanes < kThreads && lanes * VW < p.vdim) lanes *= 2;
    const uint32_t across = threadIdx.x & (lanes - 1), turn = threadIdx.x / lanes, turns = kThreads / lanes;
    for (uint32_t d0 = 0; d0 < p.vdim; d0 += lanes * VW) {
        const uint32_t d = min(d0 + across * VW, p.vdim - VW);
        float acc[REP][VW] = {};
#pragma unroll 8
        for (uint32_t k = turn; k < keys; k += turns) {
            float v[VW];
            if constexpr (VW == 4) {
                const float4 f = *reinterpret_cast<const float4 *>(V + (int64_t)k * p.vdim + d);
                v[0] = f.x, v[1] = f.y, v[2] = f.z, v[3] = f.w;
            } else {
                v[0] = V[(int64_t)k * p.vdim + d];
            }
#pragma unroll
            for (int o = 0; o < REP; o++) {
                if (o >= (int)nh) break;
                const float w = wt[o * kSeg + k];
#pragma unroll
                for (int e = 0; e < VW; e++) acc[o][e] = fmaf(w, v[e], acc[o][e]);
            }
        }
#pragma unroll
        for (int o = 0; o < REP; o++)
#pragma unroll
            for (int e = 0; e < VW; e++) red[(o * VW + e) * kThreads + threadIdx.x] = acc[o][e];
        __syncthreads();
        const uint32_t cols = min(lanes * VW, p.vdim - d0);
        for (uint32_t i = threadIdx.x; i < nh * cols; i += kThreads) {
            const uint32_t o = i / cols, c = i - o * cols;
            float sum = 0.0f;
            for (uint32_t t = 0; t < turns; t++) sum += red[(o * VW + c % VW) * kThreads + t * lanes + c / VW];
            parts[(((int64_t)blockIdx.z * nseg + seg) * p.heads + h0 + o) * p.vdim + d0 + c] = sum;
        }
        __syncthreads();
    }
}

// ---- prompts ---------------------------------------------------------------------------------------------------------
// The 16x16x4 instruction takes A[i = lane % 16][k = lane / 16], B[k = lane / 16][j = lane % 16] and leaves
// C[4 (lane / 16) + r][lane % 16] in register r.  The order of k inside a product is free: lane group g supplies
// k = 16 c + 4 g + t to the t-th of four instructions, for A and B alike.
constexpr int kTileWaves = 8;
constexpr uint32_t kRowsT = 16, kKeysT = 16;
constexpr uint32_t kRowPitch = kKeysT + 4;                // floats; 16-byte reads of 16 rows cover all banks
constexpr uint32_t kHeadPitch = kRowsT * kRowPitch + 4;   // heads four apart lie 16 banks apart
constexpr float kSlack = 24.0f;                           // a row's `top` moves when a score exceeds it by more

__device__ __forceinline__ f32x4 mfma(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// Queries of 16 rows, zero beyond a row's end.
template <int DT> __device__ __forceinline__ void load_q(const AttentionPlan &p, const float *q, uint32_t b, uint32_t s0, uint32_t li, uint32_t lg, uint32_t h, f32x4 (&f)[DT]) {
    const uint32_t s = min(s0 + li, p.S - 1);
    const float *row = q + (((int64_t)b * p.S + s) * p.heads + h) * p.dim;
#pragma unroll
    for (int c = 0; c < DT; c++) {
        const uint32_t d = 16 * c + 4 * lg;
        f[c] = *reinterpret_cast<const f32x4 *>(row + min(d, p.dim - 4));
#pragma unroll
        for (int t = 0; t < 4; t++) f[c][t] = d < p.dim ? f[c][t] : 0.0f;
    }
}
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

// DT / VT: 16-wide pieces of a key / a value row (EXACT: without a rest).  QREG: the queries stay in registers; else they are
// read for every key tile.  SHARED: a wave's heads have one kv head; its next keys and values are asked for as soon as the
// registers of these are free.  A wave whose heads are not all there computes its last one again in their place: their rows of
// the buffers meet zeros in the mixing, and nobody stores what they come to.
template <int HPW, int DT, int VT, bool QREG, bool EXACT, bool SHARED>
__global__ __launch_bounds__(kTileWaves * 64) void attention_mixed_tiles_kernel(const AttentionPlan p, const float *__restrict__ q, const uint32_t tiles, const uint32_t splits,
                                                                                float *__restrict__ dst, float2 *__restrict__ stats) {
    extern __shared__ float lds[]; // three buffers of scores [heads rounded up to 16][16][16], talk [heads rounded up][the same + 4]
    constexpr int RT = (HPW * kTileWaves + 15) / 16; // row tiles of the mixing product: the heads rounded up to 16
    constexpr uint32_t BUFFER = RT * 16 * kHeadPitch, TALK = RT * 16 + 4;
    // (where registers are short keys or values are asked for when they are needed)
    constexpr bool TIGHT = HPW * VT + (QREG ? HPW * DT : DT) + DT + VT > 40, AHEAD_K = SHARED && QREG, AHEAD_V = SHARED && !TIGHT;
    const uint32_t wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, li = lane & 15, lg = lane >> 4;
    const uint32_t tile = tiles - 1 - blockIdx.x / splits /* the last rows see the most keys: first */, split = blockIdx.x % splits, b = blockIdx.y, s0 = tile * kRowsT;
    const uint32_t h0 = wave * HPW, rep = p.heads / p.kv_heads;
    const uint32_t first_row = p.cached + s0, last_row = p.cached + min(s0 + kRowsT, p.S) - 1, last = p.cached + p.S - 1;
    uint32_t lo = first_visible(p, first_row);
    const uint32_t ntiles = (last_row + 1 - lo + kKeysT - 1) / kKeysT, per = (ntiles + splits - 1) / splits;
    const uint32_t from = min(ntiles, split * per), n = min(ntiles, from + per) - from;
    lo += from * kKeysT;

    f32x4 qf[QREG ? HPW : 1][DT], out[HPW][VT];
    float top[HPW], l[HPW]; // of row li, l of this lane's keys
    float *talk = lds + 3 * BUFFER;
    auto head_of = [&](int i) { return min(h0 + i, p.heads - 1); };
#pragma unroll
    for (int i = 0; i < HPW; i++) {
        if constexpr (QREG) load_q<DT>(p, q, b, s0, li, lg, head_of(i), qf[i]);
        top[i] = p.zero_sink ? 0.0f : kNone;
        l[i] = 0.0f;
#pragma unroll
        for (int c = 0; c < VT; c++) out[i][c] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    }
    for (uint32_t i = threadIdx.x; i < RT * 16 * RT * 16; i += kTileWaves * 64) {
        const uint32_t h = i / (RT * 16), g = i % (RT * 16);
        talk[h * TALK + g] = h < p.heads && g < p.heads ? p.talk[(int64_t)h * p.heads + g] : 0.0f;
    }
    for (uint32_t i = HPW * kTileWaves * kHeadPitch + threadIdx.x; i < BUFFER; i += kTileWaves * 64) // rows that no wave writes
        lds[i] = lds[BUFFER + i] = lds[2 * BUFFER + i] = 0.0f;
    __syncthreads();
    f32x4 k[DT];
    float v[4][VT];
    const uint32_t koff = EXACT ? 4 * lg : 0;
    auto load_k = [&](uint32_t g, uint32_t key) {
        const float *base = p.keys + ((int64_t)b * p.kv_heads + g) * p.k_block + (int64_t)key * p.dim; // (the same for the whole wave)
        const uint32_t row = min(li, last - key) * p.dim + koff;
#pragma unroll
        for (int c = 0; c < DT; c++) k[c] = *reinterpret_cast<const f32x4 *>(base + (row + (EXACT ? 16 * c : min(16 * c + 4 * lg, p.dim - 4)))); // (clamped: the query is zero there)
    };
    auto load_v = [&](uint32_t g, uint32_t key) {
        const float *base = p.values + ((int64_t)b * p.kv_heads + g) * p.v_block + (int64_t)key * p.vdim;
#pragma unroll
        for (int t = 0; t < 4; t++) {
            const uint32_t row = min(4 * lg + t, last - key) * p.vdim + (EXACT ? li : 0);
#pragma unroll
            for (int c = 0; c < VT; c++) v[t][c] = base[row + (EXACT ? 16 * c : min(16 * c + li, p.vdim - 1))]; // (clamped: columns that nobody stores)
        }
    };
    uint32_t b0 = 0, b1 = 2 * BUFFER, b2 = BUFFER; // buffers of this iteration's scores, mixing, values
    // scores of key tile `it`, mixing of the one before, soft-max and values of the one before that
    auto step = [&](uint32_t it, auto do_s, auto do_m, auto do_v) {
        const uint32_t js = lo + it * kKeysT, jv = lo + (it - 2) * kKeysT;
        f32x4 x[HPW];
        if constexpr (do_v) {
#pragma unroll
            for (int i = 0; i < HPW; i++) x[i] = *reinterpret_cast<const f32x4 *>(lds + b2 + (h0 + i) * kHeadPitch + li * kRowPitch + 4 * lg);
        }
        if constexpr (do_s) { // scores of this wave's heads (of keys that a row does not see as well)
#pragma unroll
            for (int i = 0; i < HPW; i++) {
                if (!SHARED || (!AHEAD_K && i == 0)) load_k(head_of(i) / rep, js);
                if constexpr (!QREG) load_q<DT>(p, q, b, s0, li, lg, head_of(i), qf[0]);
                f32x4 a = scores<DT>(qf[QREG ? i : 0], k);
                if (p.bias) {
                    const float slope = slope_of(head_of(i), p.heads), d = (float)(int)(first_row + 4 * lg - js - li);
#pragma unroll
                    for (int r = 0; r < 4; r++) a[r] = fmaf(-slope, d + (float)r, a[r]);
                }
                float *w = lds + b0 + (h0 + i) * kHeadPitch + li;
#pragma unroll
                for (int r = 0; r < 4; r++) w[(4 * lg + r) * kRowPitch] = a[r];
                if constexpr (TIGHT) __builtin_amdgcn_sched_barrier(0); // (one head's queries at a time)
            }
            if constexpr (AHEAD_K) load_k(head_of(0) / rep, lo + min(it + 1, n - 1) * kKeysT);
        }
        if constexpr (do_m) { // talk [heads, heads] . scores [heads, 256 columns]: a wave owns whole columns and writes them back in place
            constexpr int E = kRowsT / kTileWaves;
            float *w = lds + b1 + wave * E * kRowPitch + li;
            f32x4 acc[E][RT];
#pragma unroll
            for (int e = 0; e < E; e++)
#pragma unroll
                for (int a = 0; a < RT; a++) acc[e][a] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int c = 0; c < RT; c++) {
                f32x4 f[RT];
#pragma unroll
                for (int a = 0; a < RT; a++) f[a] = *reinterpret_cast<const f32x4 *>(talk + (16 * a + li) * TALK + 16 * c + 4 * lg);
#pragma unroll
                for (int t = 0; t < 4; t++)
#pragma unroll
                    for (int e = 0; e < E; e++) {
                        const float y = w[(16 * c + 4 * lg + t) * kHeadPitch + e * kRowPitch];
#pragma unroll
                        for (int a = 0; a < RT; a++) acc[e][a] = mfma(f[a][t], y, acc[e][a]);
                    }
            }
#pragma unroll
            for (int e = 0; e < E; e++)
#pragma unroll
                for (int a = 0; a < RT; a++)
#pragma unroll
                    for (int r = 0; r < 4; r++) w[(16 * a + 4 * lg + r) * kHeadPitch + e * kRowPitch] = acc[e][a][r];
        }
        if constexpr (do_v) { // mixed scores -> weights . values; a lane has four keys of row li
            const bool whole = jv + kKeysT - 1 <= first_row && (!p.window || last_row - jv < p.window);
            const int32_t d0 = (int32_t)(first_row + li) - (int32_t)(jv + 4 * lg);
            bool moves = false;
#pragma unroll
            for (int i = 0; i < HPW; i++)
#pragma unroll
                for (int t = 0; t < 4; t++) {
                    x[i][t] = whole || (d0 >= t && (!p.window || (uint32_t)(d0 - t) < p.window)) ? x[i][t] * kLog2e : -INFINITY;
                    moves = moves || x[i][t] - top[i] > kSlack;
                }
            if (__any(moves)) {
#pragma unroll
                for (int i = 0; i < HPW; i++) {
                    float up = fmaxf(fmaxf(x[i][0], x[i][1]), fmaxf(x[i][2], x[i][3]));
                    up = fmaxf(up, __shfl_xor(up, 16, 64));
                    up = fmaxf(top[i], fmaxf(up, __shfl_xor(up, 32, 64)));
                    const float f = __builtin_amdgcn_exp2f(top[i] - up);
                    top[i] = up;
                    l[i] *= f;
#pragma unroll
                    for (int r = 0; r < 4; r++) {
                        const float fr = __shfl(f, 4 * lg + r, 64);
#pragma unroll
                        for (int c = 0; c < VT; c++) out[i][c][r] *= fr;
                    }
                }
            }
#pragma unroll
            for (int i = 0; i < HPW; i++) {
                if (!SHARED || (!AHEAD_V && i == 0)) load_v(head_of(i) / rep, jv);
#pragma unroll
                for (int t = 0; t < 4; t++) x[i][t] = __builtin_amdgcn_exp2f(x[i][t] - top[i]);
                l[i] += (x[i][0] + x[i][1]) + (x[i][2] + x[i][3]);
#pragma unroll
                for (int t = 0; t < 4; t++)
#pragma unroll
                    for (int c = 0; c < VT; c++) out[i][c] = mfma(x[i][t], v[t][c], out[i][c]);
                if constexpr (TIGHT) __builtin_amdgcn_sched_barrier(0);
            }
            if constexpr (AHEAD_V) load_v(head_of(0) / rep, min(jv + kKeysT, lo + (n - 1) * kKeysT));
        }
        // one barrier for what this wave has read and written in LDS; loads from memory stay on their way
        asm volatile("" ::: "memory");
        __builtin_amdgcn_s_waitcnt(0xC07F); // lgkmcnt(0)
        __builtin_amdgcn_s_barrier();
        asm volatile("" ::: "memory");
        const uint32_t t = b2;
        b2 = b1;
        b1 = b0;
        b0 = t;
    };
    if (n) { // (an empty part of the keys: nothing)
        const std::true_type yes{};
        const std::false_type no{};
        if constexpr (AHEAD_K) load_k(head_of(0) / rep, lo);
        if constexpr (AHEAD_V) load_v(head_of(0) / rep, lo);
        step(0, yes, no, no);
        if (n > 1) step(1, yes, yes, no);
        for (uint32_t it = 2; it < n; it++) step(it, yes, yes, yes);
        if (n == 1) step(1, no, yes, no);
        else step(n, no, yes, yes);
        step(n + 1, no, no, yes);
    }
    const uint64_t rows = (uint64_t)p.B * p.S;
#pragma unroll
    for (int i = 0; i < HPW; i++) {
        const uint32_t h = h0 + i;
        if (h >= p.heads) break;
        float sum = l[i];
        sum += __shfl_xor(sum, 16, 64);
        sum += __shfl_xor(sum, 32, 64);
        if (splits > 1) {
            if (lg == 0 && s0 + li < p.S) stats[(split * rows + (uint64_t)b * p.S + s0 + li) * p.heads + h] = make_float2(top[i], sum);
            sum = 1.0f;
        } else if (p.zero_sink) {
            sum += __builtin_amdgcn_exp2f(-top[i]);
        }
        const float inv = 1.0f / sum;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const float f = __shfl(inv, 4 * lg + r, 64);
            const uint32_t s = s0 + 4 * lg + r;
            if (s >= p.S) continue;
            float *row = dst + ((split * rows + (uint64_t)b * p.S + s) * p.heads + h) * p.vdim + li;
#pragma unroll
            for (int c = 0; c < VT; c++)
                if (EXACT || 16 * c + li < p.vdim) row[16 * c] = out[i][c][r] * f;
        }
    }
}

// ---- a few new tokens ------------------------------------------------------------------------------------------------
// Keys are taken in chunks of `chunk`, a workgroup takes `chunks` of them.  Their keys and values are asked for first and
// arrive while the queries are prepared: four lanes share a key of a kv head (PI such keys per four lanes, DQ 16-byte pieces
// per lane), a thread has four columns of a kv head's values (for every turns-th key of the chunk).
constexpr uint32_t kMaxChunk = 64, kValuesAhead = 8;
struct StepLds { // floats
    uint32_t q, fresh, talk, raw, mixed, state, total;
};
__host__ __device__ inline StepLds step_lds(uint32_t S, uint32_t heads, uint32_t kv_heads, uint32_t dim, uint32_t chunk, uint32_t vdim) {
    StepLds o{};
    uint32_t at = 0;
    auto take = [&](uint32_t n) {
        const uint32_t r = at;
        at += (n + 3) / 4 * 4;
        return r;
    };
    o.q = take(heads * dim);
    o.fresh = take(kv_heads * dim * S); // new keys
    o.talk = take(heads * heads);
    o.raw = take(heads * (chunk + 1));
    o.mixed = take(heads * (chunk + 1));
    o.state = take(3 * heads);          // top, sum, what the results so far are multiplied by
    if (o.q + heads * vdim > at) at = o.q + heads * vdim; // (at the end the results of turns meet from `q` on)
    o.total = at;
    return o;
}

template <int REP, int DQ, int PI>
__global__ __launch_bounds__(kThreads, REP <= 4 ? 3 : 2) void attention_mixed_step_kernel(const AttentionPlan p, const uint32_t chunk, const uint32_t chunks, float *__restrict__ parts,
                                                                        float2 *__restrict__ stats) {
    extern __shared__ float lds[];
    const uint32_t rep = p.heads / p.kv_heads, seg = blockIdx.x, nseg = gridDim.x, r = blockIdx.y, b = r / p.S, s = r - b * p.S;
    const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63, pitch = chunk + 1, sub = threadIdx.x & 3;
    const StepLds at = step_lds(p.S, p.heads, p.kv_heads, p.dim, chunk, p.vdim);
    const uint32_t first = first_visible(p, p.cached + s) + seg * chunk * chunks, hi = p.cached + s + 1, end = min(hi, first + chunk * chunks);
    const uint32_t vec = p.vdim / 4, cols = p.kv_heads * vec, turns = max(1u, kThreads / cols);
    const uint32_t mine = threadIdx.x % cols, my_turn = threadIdx.x / cols; // (more columns than threads: turns 1, a second round)
    const bool has_values = cols > kThreads || my_turn < turns;
    f32x4 k[PI][DQ], v[kValuesAhead];
    auto key_of = [&](uint32_t j0, int i, uint32_t *g, uint32_t *key) {
        const uint32_t pair = (threadIdx.x >> 2) + i * (kThreads / 4);
        *g = min(pair / chunk, p.kv_heads - 1);
        *key = pair - pair / chunk * chunk;
        return pair < chunk * p.kv_heads;
    };
    // (rows that are not there or not in the cache are clamped into it: what they hold is replaced or hidden)
    auto ask_keys = [&](uint32_t j0) {
#pragma unroll
        for (int i = 0; i < PI; i++) {
            uint32_t g, key;
            key_of(j0, i, &g, &key);
            const float *src = p.keys + ((int64_t)b * p.kv_heads + g) * p.k_block + (int64_t)min(j0 + key, p.cached ? p.cached - 1 : 0) * p.dim;
#pragma unroll
            for (int d = 0; d < DQ; d++) k[i][d] = *reinterpret_cast<const f32x4 *>(src + min((uint32_t)(d * 16 + sub * 4), p.dim - 4));
        }
    };
    auto value_row = [&](uint32_t j, uint32_t g) { // new ones come from the projections
        return j < p.cached ? p.values + ((int64_t)b * p.kv_heads + g) * p.v_block + (int64_t)j * p.vdim
                            : p.v.p + ((int64_t)b * p.S + (min(j, hi - 1) - p.cached)) * p.v.pitch + g * p.vdim;
    };
    auto ask_values = [&](uint32_t j0, uint32_t c) {
        const uint32_t g = min(c / vec, p.kv_heads - 1), d = (c - c / vec * vec) * 4;
#pragma unroll
        for (uint32_t e = 0; e < kValuesAhead; e++)
            if (e * turns < chunk) v[e] = *reinterpret_cast<const f32x4 *>(value_row(min(j0 + my_turn % turns + e * turns, hi - 1), g) + d);
    };
    // a wave's heads: values lane and lane + 64 of each (one of a kind where a head is shorter)
    constexpr int QH = 4, QV = DQ > 4 ? 2 : 1;
    constexpr uint32_t kWaves = kThreads / 64;
    float qv[QH][QV];
    const uint32_t d0 = min(lane, p.dim - 1), d1 = min(lane + 64, p.dim - 1);
    auto ask_heads = [&](const float *src, uint32_t h0, uint32_t n) {
#pragma unroll
        for (int i = 0; i < QH; i++) {
            const float *x = src + min(h0 + i * kWaves + wave, n - 1) * p.dim;
            qv[i][0] = x[d0];
            if (QV > 1) qv[i][QV - 1] = x[d1];
        }
    };
    float2 turn[QV];
    auto ask_turn = [&](uint32_t t) {
#pragma unroll
        for (int v = 0; v < QV; v++) {
            const uint32_t d = lane + 64 * v;
            turn[v] = make_float2(1.0f, 0.0f);
            if (d < p.rot_dims) turn[v] = rotation_at(p, p.position + t, d / 2);
            if (!(d & 1)) turn[v].y = -turn[v].y;
        }
    };
    ask_heads(p.q.p + (int64_t)r * p.q.pitch, 0, p.heads);
    ask_turn(s);
    ask_keys(first);
    ask_values(first, mine);

    const uint32_t t0 = first > p.cached ? first - p.cached : 0, t1 = end > p.cached && end > first ? end - p.cached : 0; // new keys [t0, t1)
    for (uint32_t i = threadIdx.x; i < p.heads * p.heads; i += kThreads) { // (transposed: lanes side by side read other heads' columns)
        const uint32_t h = i / p.heads, g = i - h * p.heads;
        lds[at.talk + g * p.heads + h] = p.talk ? p.talk[i] : h == g ? 1.0f : 0.0f;
    }
    for (uint32_t h = threadIdx.x; h < p.heads; h += kThreads) {
        lds[at.state + h] = kNone;
        lds[at.state + p.heads + h] = 0.0f;
    }
    // the heads of a token: turned, at a mean square of one, times f
    auto put_heads = [&](uint32_t h0, uint32_t n, float f, float *dst, float *cache, int64_t cache_pitch) {
#pragma unroll
        for (int i = 0; i < QH; i++) {
            const uint32_t h = h0 + i * kWaves + wave;
            float x[QV], m = 0.0f;
#pragma unroll
            for (int v = 0; v < QV; v++) {
                x[v] = fmaf(qv[i][v], turn[v].x, __shfl_xor(qv[i][v], 1, 64) * turn[v].y);
                if (lane + 64 * v < p.dim) m = fmaf(x[v], x[v], m);
            }
            float g = f;
            if (p.unit_heads) g /= sqrtf(wave_total(m) / (float)p.dim + p.eps);
#pragma unroll
            for (int v = 0; v < QV; v++)
                if (h < n && lane + 64 * v < p.dim) {
                    dst[h * p.dim + lane + 64 * v] = x[v] * g;
                    if (cache) cache[h * cache_pitch + lane + 64 * v] = x[v] * g;
                }
        }
    };
    float temp = p.scale;
    if (p.temp_every) temp *= 1.0f + p.temp_coef * logf((float)((p.position + s + 1) / p.temp_every + 1));
    for (uint32_t h0 = 0; h0 < p.heads; h0 += QH * kWaves) {
        if (h0) ask_heads(p.q.p + (int64_t)r * p.q.pitch, h0, p.heads);
        put_heads(h0, p.heads, temp, lds + at.q, nullptr, 0);
    }
    for (uint32_t t = t0; t < t1; t++) {
        if (t != s || t > t0) ask_turn(t);
        float *cache = t == s ? p.keys + (int64_t)b * p.kv_heads * p.k_block + (int64_t)(p.cached + t) * p.dim : nullptr; // its own workgroup's
        for (uint32_t h0 = 0; h0 < p.kv_heads; h0 += QH * kWaves) {
            ask_heads(p.k.p + ((int64_t)b * p.S + t) * p.k.pitch, h0, p.kv_heads);
            put_heads(h0, p.kv_heads, 1.0f, lds + at.fresh + t * p.kv_heads * p.dim, cache, p.k_block);
        }
    }
    if (t1 == s + 1 && t0 <= s) // the last segment: this token's values
        for (uint32_t i = threadIdx.x; i < p.kv_heads * p.vdim; i += kThreads) {
            const uint32_t g = i / p.vdim, d = i - g * p.vdim;
            p.values[((int64_t)b * p.kv_heads + g) * p.v_block + (int64_t)(p.cached + s) * p.vdim + d] = p.v.p[(int64_t)r * p.v.pitch + i];
        }
    __syncthreads();
    f32x4 acc[REP] = {};
    for (uint32_t j0 = first; j0 < end; j0 += chunk) {
        const uint32_t keys = min(chunk, end - j0);
#pragma unroll
        for (int i = 0; i < PI; i++) {
            uint32_t g, key;
            const bool there = key_of(j0, i, &g, &key);
            const uint32_t j = j0 + key;
            if (there && key < keys && j >= p.cached) {
#pragma unroll
                for (int d = 0; d < DQ; d++)
                    k[i][d] = *reinterpret_cast<const f32x4 *>(lds + at.fresh + ((j - p.cached) * p.kv_heads + g) * p.dim + min((uint32_t)(d * 16 + sub * 4), p.dim - 4));
            }
            for (uint32_t h0 = 0; h0 < rep; h0 += REP) {
#pragma unroll
                for (int h = 0; h < REP; h++) {
                    const uint32_t hh = g * rep + min(h0 + h, rep - 1);
                    const float *qh = lds + at.q + hh * p.dim;
                    float x = 0.0f;
#pragma unroll
                    for (int d = 0; d < DQ; d++) {
                        const uint32_t e = d * 16 + sub * 4;
                        const f32x4 qv = *reinterpret_cast<const f32x4 *>(qh + min(e, p.dim - 4));
                        const float y = fmaf(k[i][d][0], qv[0], fmaf(k[i][d][1], qv[1], fmaf(k[i][d][2], qv[2], k[i][d][3] * qv[3])));
                        x += e < p.dim ? y : 0.0f;
                    }
                    x += __shfl_xor(x, 1, 64);
                    x += __shfl_xor(x, 2, 64);
                    if (sub == 0 && there && h0 + h < rep) {
                        if (p.bias) x -= slope_of(hh, p.heads) * (float)(int)(p.cached + s - j);
                        lds[at.raw + hh * pitch + key] = key < keys ? x : 0.0f;
                    }
                }
            }
        }
        if (j0 + chunk < end) ask_keys(j0 + chunk); // on their way meanwhile
        __syncthreads();
        for (uint32_t i = threadIdx.x; i < p.heads * chunk; i += kThreads) {
            const uint32_t key = i / p.heads, h = i - key * p.heads;
            float w = 0.0f;
#pragma unroll 8
            for (uint32_t g = 0; g < p.heads; g++) w = fmaf(lds[at.talk + g * p.heads + h], lds[at.raw + g * pitch + key], w);
            lds[at.mixed + h * pitch + key] = key < keys ? w * kLog2e : -INFINITY;
        }
        __syncthreads();
        // (lanes side by side take a head each, a run of the chunk's keys every one)
        for (uint32_t i = threadIdx.x; i < p.heads * 4; i += kThreads) {
            const uint32_t h = i / 4;
            float *x = lds + at.mixed + h * pitch;
            const float top = lds[at.state + h];
            float m = top, l = 0.0f;
            for (uint32_t key = i % 4; key < chunk; key += 4) m = fmaxf(m, x[key]);
            m = fmaxf(m, __shfl_xor(m, 1, 64));
            m = fmaxf(m, __shfl_xor(m, 2, 64));
            for (uint32_t key = i % 4; key < chunk; key += 4) {
                const float e = __builtin_amdgcn_exp2f(x[key] - m);
                x[key] = e;
                l += e;
            }
            l += __shfl_xor(l, 1, 64);
            l += __shfl_xor(l, 2, 64);
            if (i % 4 == 0) {
                const float f = __builtin_amdgcn_exp2f(top - m);
                lds[at.state + h] = m;
                lds[at.state + p.heads + h] = fmaf(lds[at.state + p.heads + h], f, l);
                lds[at.state + 2 * p.heads + h] = f;
            }
        }
        __syncthreads();
        // a thread's columns: results of this chunk for one kv head's query heads, REP at a time
        auto weigh = [&](uint32_t c, uint32_t h0, f32x4(&o)[REP]) {
            const uint32_t g = c / vec;
#pragma unroll
            for (uint32_t e = 0; e < kValuesAhead; e++) {
                const uint32_t key = my_turn % turns + e * turns;
                if (key >= keys) break;
#pragma unroll
                for (int h = 0; h < REP; h++) {
                    const float w = lds[at.mixed + (g * rep + min(h0 + h, rep - 1)) * pitch + key];
#pragma unroll
                    for (int d = 0; d < 4; d++) o[h][d] = fmaf(w, v[e][d], o[h][d]);
                }
            }
        };
        if (has_values) {
#pragma unroll
            for (int h = 0; h < REP; h++) acc[h] *= lds[at.state + 2 * p.heads + (mine / vec) * rep + min((uint32_t)h, rep - 1)];
            weigh(mine, 0, acc);
        }
        if (j0 + chunk < end) {
            ask_values(j0 + chunk, mine);
            __syncthreads();
        }
    }
    __syncthreads();
    for (uint32_t h = threadIdx.x; h < p.heads; h += kThreads) stats[((int64_t)r * nseg + seg) * p.heads + h] = make_float2(lds[at.state + h], lds[at.state + p.heads + h]);
    float *dst = parts + ((int64_t)r * nseg + seg) * p.heads * p.vdim;
    if (turns > 1) { // the turns' results meet in LDS, from the queries' place on, one turn after the other
        for (uint32_t t = 0; t < turns; t++) {
            __syncthreads();
            if (my_turn == t) {
#pragma unroll
                for (int h = 0; h < REP; h++) {
                    if (h >= (int)rep) break;
                    f32x4 *o = reinterpret_cast<f32x4 *>(lds + at.q + ((mine / vec) * rep + h) * p.vdim + (mine % vec) * 4);
                    *o = t ? *o + acc[h] : acc[h];
                }
            }
        }
        __syncthreads();
        for (uint32_t i = threadIdx.x; i < p.heads * vec; i += kThreads) *reinterpret_cast<f32x4 *>(dst + 4 * i) = *reinterpret_cast<const f32x4 *>(lds + at.q + 4 * i);
    } else if (has_values) {
#pragma unroll
        for (int h = 0; h < REP; h++)
            if (h < (int)rep) *reinterpret_cast<f32x4 *>(dst + ((mine / vec) * rep + h) * p.vdim + (mine % vec) * 4) = acc[h];
    }
}

int launched(const char *what) {
    const hipError_t e = hipGetLastError();
    return e == hipSuccess ? CG_OK : hip_fail(e, what);
}
constexpr size_t kMaxLds = 160 << 10;
int allow_lds(const void *kernel, size_t bytes) {
    if (bytes > kMaxLds) return fail(CG_ERR_UNSUPPORTED, "block_attention: heads or sizes beyond what the kernels hold");
    if (bytes <= (64 << 10)) return CG_OK;
    const hipError_t e = hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
    return e == hipSuccess ? CG_OK : hip_fail(e, "hipFuncSetAttribute");
}

struct Scratch {
    cg_backend *be;
    void *p = nullptr;
    size_t cls = 0;
    explicit Scratch(cg_backend *b) : be(b) {}
    int get(size_t bytes) { return be->pool.alloc(bytes ? bytes : 4, &p, &cls); }
    ~Scratch() {
        if (p) be->pool.free(p, cls);
    }
};

// few segments of many rows: a thread per four results (vdim a multiple of 4) or one
template <int VW>
__global__ __launch_bounds__(kThreads) void attention_merge_rows_kernel(const float *__restrict__ parts, const float2 *__restrict__ stats, const uint32_t segs,
                                                                        const uint64_t row_pitch, const uint64_t seg_pitch, const uint32_t heads, const uint32_t vdim,
                                                                        const bool sink, const uint64_t total, float *__restrict__ out) {
    const uint64_t i = ((uint64_t)blockIdx.x * kThreads + threadIdx.x) * VW;
    if (i >= total) return;
    const uint32_t n = heads * vdim;
    const uint64_t row = i / n;
    const uint32_t c = (uint32_t)(i - row * n);
    const float *p = parts + row * row_pitch * vdim + c;
    const float2 *st = stats + row * row_pitch + c / vdim;
    float m = sink ? 0.0f : kNone, l = 0.0f, o[VW] = {};
    for (uint32_t k = 0; k < segs; k++) m = fmaxf(m, st[k * seg_pitch].x);
    if (sink) l = __builtin_amdgcn_exp2f(-m);
    for (uint32_t k = 0; k < segs; k++) {
        const float2 t = st[k * seg_pitch];
        const float f = __builtin_amdgcn_exp2f(t.x - m);
        l = fmaf(t.y, f, l);
        if constexpr (VW == 4) {
            const float4 v = *reinterpret_cast<const float4 *>(p + k * seg_pitch * vdim);
            o[0] = fmaf(v.x, f, o[0]), o[1] = fmaf(v.y, f, o[1]), o[2] = fmaf(v.z, f, o[2]), o[3] = fmaf(v.w, f, o[3]);
        } else {
            o[0] = fmaf(p[k * seg_pitch * vdim], f, o[0]);
        }
    }
    const float inv = 1.0f / l;
    if constexpr (VW == 4) *reinterpret_cast<float4 *>(out + i) = make_float4(o[0] * inv, o[1] * inv, o[2] * inv, o[3] * inv);
    else out[i] = o[0] * inv;
}

void merge(cg_backend *be, const AttentionPlan &p, const float *parts, const float2 *stats, uint32_t segs, uint64_t row_pitch, uint64_t seg_pitch, uint32_t rows, float *out) {
    const uint32_t n = p.heads * p.vdim;
    if (segs <= 8) {
        const uint64_t total = (uint64_t)rows * n;
        if (p.vdim % 4 == 0)
            hipLaunchKernelGGL((attention_merge_rows_kernel<4>), dim3((uint32_t)((total / 4 + kThreads - 1) / kThreads)), dim3(kThreads), 0, be->stream, parts, stats, segs, row_pitch,
                               seg_pitch, p.heads, p.vdim, p.zero_sink, total, out);
        else
            hipLaunchKernelGGL((attention_merge_rows_kernel<1>), dim3((uint32_t)((total + kThreads - 1) / kThreads)), dim3(kThreads), 0, be->stream, parts, stats, segs, row_pitch,
                               seg_pitch, p.heads, p.vdim, p.zero_sink, total, out);
        return;
    }
    for (uint32_t r0 = 0; r0 < rows; r0 += 65535) {
        const uint32_t nr = std::min(rows - r0, 65535u);
        hipLaunchKernelGGL(attention_merge_kernel, dim3((n + 63) / 64, nr), dim3(kMergeWaves * 64), 0, be->stream, parts + (uint64_t)r0 * row_pitch * p.vdim,
                           stats + (uint64_t)r0 * row_pitch, segs, row_pitch, seg_pitch, p.heads, p.vdim, p.zero_sink, out + (uint64_t)r0 * n);
    }
}

template <int REP, int VW>
int mixed_rows(cg_backend *be, const AttentionPlan &p, uint32_t row0, uint32_t rows, uint32_t nseg, const float *scores, float *parts, float2 *stats) {
    const uint32_t rep = p.heads / p.kv_heads, groups = (rep + REP - 1) / REP, slots = p.talk ? p.heads : REP;
    const size_t lds = (size_t)mixed_floats(REP, slots, VW) * 4;
    if (int rc = allow_lds(reinterpret_cast<const void *>(&attention_mixed_rows_kernel<REP, VW>), lds)) return rc;
    hipLaunchKernelGGL((attention_mixed_rows_kernel<REP, VW>), dim3(nseg, p.kv_heads * groups, rows), dim3(kThreads), lds, be->stream, p, row0, nseg, scores, parts, stats);
    merge(be, p, parts, stats, nseg, (uint64_t)nseg * p.heads, p.heads, rows, p.out + (uint64_t)row0 * p.heads * p.vdim);
    return launched("attention_mixed_rows");
}

template <int HPW, int DT, int VT, bool QREG, bool EXACT, bool SHARED>
int launch_tiles(cg_backend *be, const AttentionPlan &p, const float *q, uint32_t splits, float *dst, float2 *stats) {
    const uint32_t tiles = (p.S + kRowsT - 1) / kRowsT;
    const size_t h16 = (HPW * kTileWaves + 15) / 16 * 16, lds = (3 * h16 * kHeadPitch + h16 * (h16 + 4)) * 4;
    if (int rc = allow_lds(reinterpret_cast<const void *>(&attention_mixed_tiles_kernel<HPW, DT, VT, QREG, EXACT, SHARED>), lds)) return rc;
    hipLaunchKernelGGL((attention_mixed_tiles_kernel<HPW, DT, VT, QREG, EXACT, SHARED>), dim3(tiles * splits, p.B), dim3(kTileWaves * 64), lds, be->stream, p, q, tiles, splits, dst,
                       stats);
    return CG_OK;
}
template <int HPW, int DT, int VT, bool QREG, bool EXACT = false>
int run_tiles(cg_backend *be, const AttentionPlan &p, const float *q, uint32_t splits, float *dst, float2 *stats) {
    if (HPW == 1 || p.heads / p.kv_heads % HPW == 0) return launch_tiles<HPW, DT, VT, QREG, EXACT, true>(be, p, q, splits, dst, stats);
    return launch_tiles<HPW, DT, VT, QREG, EXACT, HPW == 1>(be, p, q, splits, dst, stats);
}
template <int HPW> int run_tiles(cg_backend *be, const AttentionPlan &p, const float *q, uint32_t splits, float *dst, float2 *stats) {
    const uint32_t d = p.dim, v = p.vdim;
    if (d == 64 && v == 64) return run_tiles<HPW, 4, 4, true, true>(be, p, q, splits, dst, stats);
    if (d == 128 && v == 128) return run_tiles<HPW, 8, 8, (HPW < 4), true>(be, p, q, splits, dst, stats);
    if (d <= 32 && v <= 32) return run_tiles<HPW, 2, 2, true>(be, p, q, splits, dst, stats);
    if (d <= 64 && v <= 64) return run_tiles<HPW, 4, 4, true>(be, p, q, splits, dst, stats);
    if (d <= 64 && v <= 96) return run_tiles<HPW, 4, 6, (HPW < 4)>(be, p, q, splits, dst, stats);
    if (d <= 96 && v <= 96) return run_tiles<HPW, 6, 6, (HPW < 4)>(be, p, q, splits, dst, stats);
    return run_tiles<HPW, 8, 8, (HPW < 4)>(be, p, q, splits, dst, stats);
}

} // namespace

int launch_mixed_rows(cg_backend *be, const AttentionPlan &p, uint32_t row0, uint32_t rows, uint32_t nseg, const float *scores, float *parts, float2 *part_stats) {
    const uint32_t rep = p.heads / p.kv_heads;
    const bool vec = p.vdim % 4 == 0; // (cache rows begin at multiples of their length: 16-byte loads then)
#define CG_ROWS(R) (vec ? mixed_rows<R, 4>(be, p, row0, rows, nseg, scores, parts, part_stats) : mixed_rows<R, 1>(be, p, row0, rows, nseg, scores, parts, part_stats))
    return rep <= 1 ? CG_ROWS(1) : rep <= 2 ? CG_ROWS(2) : rep <= 4 ? CG_ROWS(4) : CG_ROWS(8);
#undef CG_ROWS
}

int launch_mixed_tiles(cg_backend *be, const AttentionPlan &p, const float *q) {
    if (p.S <= kFewRows || p.heads > 32 || p.dim % 4 || p.dim > 128 || p.vdim > 128 || p.B > 65535 || !p.talk) return kDeclined;
    const uint64_t n = (uint64_t)p.B * p.S * p.heads * p.vdim;
    const uint32_t tiles = (p.S + kRowsT - 1) / kRowsT, keys = p.cached + p.S, most = p.window ? std::min(p.window + kRowsT, keys) : keys;
    // too few row tiles for the device: their keys are cut over up to 4 workgroups, each with at least 8 key tiles
    const uint32_t want = (uint32_t)(2 * be->compute_units) / std::max(1u, tiles * p.B);
    const uint32_t splits = std::max(1u, std::min(std::min(4u, want), most / (8 * kKeysT)));
    Scratch parts(be), stats(be);
    if (splits > 1) {
        if (int rc = parts.get((size_t)n * splits * 4)) return rc;
        if (int rc = stats.get((size_t)p.B * p.S * p.heads * splits * sizeof(float2))) return rc;
    }
    float *dst = splits > 1 ? static_cast<float *>(parts.p) : p.out;
    float2 *st = static_cast<float2 *>(stats.p);
    const int rc = p.heads <= 8    ? run_tiles<1>(be, p, q, splits, dst, st)
                   : p.heads <= 16 ? run_tiles<2>(be, p, q, splits, dst, st)
                                   : run_tiles<4>(be, p, q, splits, dst, st);
    if (rc) return rc;
    if (splits > 1) merge(be, p, dst, st, splits, p.heads, (uint64_t)p.B * p.S * p.heads, p.B * p.S, p.out);
    return launched("attention_mixed_tiles");
}

template <int REP, int DQ>
static int step_kernels(cg_backend *be, const AttentionPlan &p, uint32_t chunk, uint32_t chunks, dim3 grid, size_t lds, float *parts, float2 *stats) {
    constexpr int PI = 8 / DQ; // keys of four lanes: 8 pieces per lane
    if (int rc = allow_lds(reinterpret_cast<const void *>(&attention_mixed_step_kernel<REP, DQ, PI>), lds)) return rc;
    hipLaunchKernelGGL((attention_mixed_step_kernel<REP, DQ, PI>), grid, dim3(kThreads), lds, be->stream, p, chunk, chunks, parts, stats);
    return CG_OK;
}

int launch_mixed_step(cg_backend *be, const AttentionPlan &p) {
    const uint32_t rows = p.B * p.S, keys = p.cached + p.S, most = p.window ? std::min(p.window, keys) : keys, rep = p.heads / p.kv_heads, cols = p.kv_heads * p.vdim / 4;
    auto aligned = [](const Rows &x) { return x.pitch % 4 == 0 && (reinterpret_cast<uintptr_t>(x.p) & 15) == 0; };
    if (p.S > kFewRows || p.dim % 4 || p.vdim % 4 || rows > 65535 || p.q_norm || p.k_norm || rep > 8 || p.dim > 128 || cols > kThreads || !aligned(p.v)) return kDeclined;
    // chunks whose keys and values a workgroup holds in registers
    const uint32_t turns = std::max(1u, (uint32_t)kThreads / cols), dq = p.dim <= 32 ? 2 : p.dim <= 64 ? 4 : 8, pairs = kThreads / 4 * (8 / dq);
    if (p.kv_heads > pairs) return kDeclined;
    uint32_t chunk = kMaxChunk;
    while (chunk * p.kv_heads > pairs || chunk > turns * kValuesAhead) chunk /= 2;
    const size_t lds = (size_t)step_lds(p.S, p.heads, p.kv_heads, p.dim, chunk, p.vdim).total * 4;
    if (lds > kMaxLds / 2) return kDeclined;
    // as many workgroups as run at a time
    const uint32_t all = (most + chunk - 1) / chunk;
    const uint32_t resident = (rep <= 4 ? 3 : 2) * be->compute_units, chunks = (uint32_t)(((uint64_t)rows * all + resident - 1) / resident), nseg = (all + chunks - 1) / chunks;
    Scratch mem(be);
    const size_t n = (size_t)rows * nseg * p.heads;
    if (int rc = mem.get(n * p.vdim * 4 + n * sizeof(float2))) return rc;
    float *parts = static_cast<float *>(mem.p);
    float2 *stats = reinterpret_cast<float2 *>(parts + n * p.vdim);
    const dim3 grid(nseg, rows);
    int rc;
#define CG_STEP(R) (p.dim <= 32 ? step_kernels<R, 2>(be, p, chunk, chunks, grid, lds, parts, stats) \
                    : p.dim <= 64 ? step_kernels<R, 4>(be, p, chunk, chunks, grid, lds, parts, stats) \
                                  : step_kernels<R, 8>(be, p, chunk, chunks, grid, lds, parts, stats))
    if (rep <= 1) rc = CG_STEP(1);
    else if (rep <= 2) rc = CG_STEP(2);
    else if (rep <= 4) rc = CG_STEP(4);
    else rc = CG_STEP(8);
#undef CG_STEP
    if (rc) return rc;
    merge(be, p, parts, stats, nseg, (uint64_t)nseg * p.heads, p.heads, rows, p.out);
    return launched("attention_mixed_step");
}

} // namespace cg
