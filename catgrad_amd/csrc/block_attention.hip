// Causal attention of new tokens behind a cache, with a window, a distance bias, a query temperature, norms over whole
// projections, rotations, unit heads, a sink, and head mixing after the soft-max or before it (cg_block_attention; the latter's
// kernels are in block_attention_mixed.hip).
//
//   attention_prepare_kernel  more than a few new tokens, a workgroup per token: the query row normed and scaled, the key and
//                             value rows into the cache (then block_attention_tiles.hip, for the sizes it takes)
//   attention_turn_*_kernel   the same with rotations and unit heads
//   attention_scores_kernel   a workgroup per (token, kv head, 128 keys): scores, and their maximum and sum per head; with a
//                             few new tokens the preparation as well
//   attention_mix_kernel      the same split: soft-max weights of every head, mixed, times the values of the kv head
//   attention_sum_kernel      partial results of a token's key segments added up
#include "blocks.hpp"
#include "device_utils.hpp"

#include <algorithm>

namespace cg {
namespace {

constexpr int kThreads = 256, kWaves = 4;
constexpr uint32_t kSeg = 128; // keys of a segment

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int d = 32; d > 0; d >>= 1) v += __shfl_xor(v, d, 64);
    return v;
}
__device__ __forceinline__ float block_sum(float v, float *red) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}
__device__ __forceinline__ float slope_of(uint32_t h, uint32_t heads) { return exp2f(-8.0f * (float)(h + 1) / (float)heads); }

// Visible keys of the token in row s: [lo, hi) of the cached and new keys together.
__device__ __forceinline__ void visible(const AttentionPlan &p, uint32_t s, uint32_t *lo, uint32_t *hi) {
    const uint32_t i = p.cached + s;
    *hi = i + 1;
    *lo = p.window && i + 1 > p.window ? i + 1 - p.window : 0;
}

__global__ __launch_bounds__(kThreads) void attention_prepare_kernel(const AttentionPlan p, float *__restrict__ q) {
    __shared__ float red[kWaves];
    const uint32_t r = blockIdx.x, b = r / p.S, s = r - b * p.S;
    const uint32_t nq = p.heads * p.dim, nk = p.kv_heads * p.dim, nv = p.kv_heads * p.vdim;
    const float *qr = p.q.p + (int64_t)r * p.q.pitch, *kr = p.k.p + (int64_t)r * p.k.pitch, *vr = p.v.p + (int64_t)r * p.v.pitch;
    float mq = 0.0f, mk = 0.0f;
    if (p.q_norm)
        for (uint32_t i = threadIdx.x; i < nq; i += kThreads) mq = fmaf(qr[i], qr[i], mq);
    if (p.k_norm)
        for (uint32_t i = threadIdx.x; i < nk; i += kThreads) mk = fmaf(kr[i], kr[i], mk);
    float fq = 1.0f, fk = 1.0f;
    if (p.q_norm) fq = 1.0f / sqrtf(block_sum(mq, red) / (float)nq + p.eps);
    if (p.k_norm) fk = 1.0f / sqrtf(block_sum(mk, red) / (float)nk + p.eps);
    float temp = p.scale;
    if (p.temp_every) temp *= 1.0f + p.temp_coef * logf((float)((p.position + s + 1) / p.temp_every + 1));
    for (uint32_t i = threadIdx.x; i < nq; i += kThreads) {
        float v = qr[i];
        if (p.q_norm) v = v * fq * p.q_norm[i];
        q[(int64_t)r * nq + i] = v * temp;
    }
    float *kc = p.keys + (int64_t)b * p.kv_heads * p.k_block + (int64_t)(p.cached + s) * p.dim;
    float *vc = p.values + (int64_t)b * p.kv_heads * p.v_block + (int64_t)(p.cached + s) * p.vdim;
    for (uint32_t i = threadIdx.x; i < nk; i += kThreads) {
        const uint32_t g = i / p.dim, d = i - g * p.dim;
        float v = kr[i];
        if (p.k_norm) v = v * fk * p.k_norm[i];
        kc[(int64_t)g * p.k_block + d] = v;
    }
    for (uint32_t i = threadIdx.x; i < nv; i += kThreads) {
        const uint32_t g = i / p.vdim, d = i - g * p.vdim;
        vc[(int64_t)g * p.v_block + d] = vr[i];
    }
}

// Rows of a rotation's table: {cos, sin} of the positions first, first + step, ...
__global__ __launch_bounds__(kThreads) void rotation_table_kernel(float2 *__restrict__ t, const uint32_t rows, const uint32_t step, const uint32_t dims, const double log2_base) {
    const uint32_t i = blockIdx.x * kThreads + threadIdx.x, pairs = dims / 2;
    if (i >= rows * pairs) return;
    double a = (double)((uint64_t)(i / pairs) * step) * exp2(-2.0 * (double)(i % pairs) / (double)dims * log2_base);
    a -= 6.283185307179586 * rint(a * 0.15915494309189535);
    t[i] = make_float2((float)cos(a), (float)sin(a));
}

// The same with every head turned by its token's angles and brought to a mean square of one, a wave per head.
__global__ __launch_bounds__(kThreads) void attention_turn_kernel(const AttentionPlan p, float *__restrict__ q) {
    extern __shared__ float2 turn[]; // {cos, sin} per pair
    __shared__ float red[kWaves];
    const uint32_t r = blockIdx.x, b = r / p.S, s = r - b * p.S, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const uint32_t nq = p.heads * p.dim, nk = p.kv_heads * p.dim, nv = p.kv_heads * p.vdim;
    const float *qr = p.q.p + (int64_t)r * p.q.pitch, *kr = p.k.p + (int64_t)r * p.k.pitch, *vr = p.v.p + (int64_t)r * p.v.pitch;
    for (uint32_t i = threadIdx.x; i < p.rot_dims / 2; i += kThreads) turn[i] = rotation_at(p, p.position + s, i);
    float mq = 0.0f, mk = 0.0f;
    if (p.q_norm)
        for (uint32_t i = threadIdx.x; i < nq; i += kThreads) mq = fmaf(qr[i], qr[i], mq);
    if (p.k_norm)
        for (uint32_t i = threadIdx.x; i < nk; i += kThreads) mk = fmaf(kr[i], kr[i], mk);
    float fq = 1.0f, fk = 1.0f;
    if (p.q_norm) fq = 1.0f / sqrtf(block_sum(mq, red) / (float)nq + p.eps);
    if (p.k_norm) fk = 1.0f / sqrtf(block_sum(mk, red) / (float)nk + p.eps);
    float temp = p.scale;
    if (p.temp_every) temp *= 1.0f + p.temp_coef * logf((float)((p.position + s + 1) / p.temp_every + 1));
    __syncthreads();
    for (uint32_t h = wave; h < p.heads + p.kv_heads; h += kWaves) {
        const bool key = h >= p.heads;
        const uint32_t g = h - p.heads;
        const float *src = key ? kr + g * p.dim : qr + h * p.dim, *w = key ? p.k_norm : p.q_norm;
        if (w) w += (key ? g : h) * p.dim;
        float *dst = key ? p.keys + ((int64_t)b * p.kv_heads + g) * p.k_block + (int64_t)(p.cached + s) * p.dim : q + (int64_t)r * nq + h * p.dim;
        const float f = key ? fk : fq;
        auto plain = [&](uint32_t d) { return w ? src[d] * f * w[d] : src[d]; };
        auto value = [&](uint32_t d) {
            const float v = plain(d);
            if (d >= p.rot_dims) return v;
            const float2 cs = turn[d / 2];
            return d & 1 ? fmaf(v, cs.x, plain(d - 1) * cs.y) : fmaf(v, cs.x, -plain(d + 1) * cs.y);
        };
        const float v0 = lane < p.dim ? value(lane) : 0.0f, v1 = lane + 64 < p.dim ? value(lane + 64) : 0.0f;
        float m = fmaf(v0, v0, v1 * v1), c = key ? 1.0f : temp;
        for (uint32_t d = lane + 128; d < p.dim; d += 64) {
            const float v = value(d);
            m = fmaf(v, v, m);
        }
        if (p.unit_heads) c /= sqrtf(wave_sum(m) / (float)p.dim + p.eps);
        for (uint32_t d = lane; d < p.dim; d += 64) dst[d] = (d == lane ? v0 : d == lane + 64 ? v1 : value(d)) * c;
    }
    float *vc = p.values + (int64_t)b * p.kv_heads * p.v_block + (int64_t)(p.cached + s) * p.vdim;
    for (uint32_t i = threadIdx.x; i < nv; i += kThreads) {
        const uint32_t g = i / p.vdim, d = i - g * p.vdim;
        vc[(int64_t)g * p.v_block + d] = vr[i];
    }
}

// The same for heads of 4 * LANES values or fewer (a multiple of 4) without norms over whole projections: LANES lanes share a
// head, 64 / LANES heads a wave at a time, all of a workgroup's tokens' heads in turn.
template <int LANES> __global__ __launch_bounds__(kThreads) void attention_turn_heads_kernel(const AttentionPlan p, float *__restrict__ q) {
    const uint32_t sub = threadIdx.x % LANES, r = blockIdx.x, b = r / p.S, s = r - b * p.S, d = min(sub * 4, p.dim - 4);
    const bool there = sub * 4 < p.dim;
    float2 t0 = make_float2(1.0f, 0.0f), t1 = t0;
    if (sub * 4 < p.rot_dims) t0 = rotation_at(p, p.position + s, sub * 2);
    if (sub * 4 + 2 < p.rot_dims) t1 = rotation_at(p, p.position + s, sub * 2 + 1);
    float temp = p.scale;
    if (p.temp_every) temp *= 1.0f + p.temp_coef * logf((float)((p.position + s + 1) / p.temp_every + 1));
    const uint32_t heads = p.heads + p.kv_heads;
#pragma unroll 2
    for (uint32_t h0 = 0; h0 < heads; h0 += kThreads / LANES) { // (the same trips for every lane: the sums are over lanes)
        const uint32_t h = min(h0 + threadIdx.x / LANES, heads - 1), g = h - p.heads;
        const bool key = h >= p.heads;
        const float4 v = *reinterpret_cast<const float4 *>((key ? p.k.p + (int64_t)r * p.k.pitch + g * p.dim : p.q.p + (int64_t)r * p.q.pitch + h * p.dim) + d);
        float4 x = make_float4(fmaf(v.x, t0.x, -v.y * t0.y), fmaf(v.y, t0.x, v.x * t0.y), fmaf(v.z, t1.x, -v.w * t1.y), fmaf(v.w, t1.x, v.z * t1.y));
        float c = key ? 1.0f : temp;
        if (p.unit_heads) {
            float m = there ? fmaf(x.x, x.x, fmaf(x.y, x.y, fmaf(x.z, x.z, x.w * x.w))) : 0.0f;
#pragma unroll
            for (int e = 1; e < LANES; e <<= 1) m += __shfl_xor(m, e, 64);
            c /= sqrtf(m / (float)p.dim + p.eps);
        }
        if (!there || h0 + threadIdx.x / LANES >= heads) continue;
        float *dst = key ? p.keys + ((int64_t)b * p.kv_heads + g) * p.k_block + (int64_t)(p.cached + s) * p.dim : q + ((int64_t)r * p.heads + h) * p.dim;
        *reinterpret_cast<float4 *>(dst + d) = make_float4(x.x * c, x.y * c, x.z * c, x.w * c);
    }
    float *vc = p.values + (int64_t)b * p.kv_heads * p.v_block + (int64_t)(p.cached + s) * p.vdim;
    const float *vr = p.v.p + (int64_t)r * p.v.pitch;
    if (p.vdim % 4 == 0 && p.v.pitch % 4 == 0 && (reinterpret_cast<uintptr_t>(p.v.p) & 15) == 0) {
        for (uint32_t i = threadIdx.x; i < p.kv_heads * p.vdim / 4; i += kThreads) {
            const uint32_t g = i * 4 / p.vdim, e = i * 4 - g * p.vdim;
            *reinterpret_cast<float4 *>(vc + (int64_t)g * p.v_block + e) = *reinterpret_cast<const float4 *>(vr + 4 * i);
        }
    } else {
        for (uint32_t i = threadIdx.x; i < p.kv_heads * p.vdim; i += kThreads) {
            const uint32_t g = i / p.vdim, e = i - g * p.vdim;
            vc[(int64_t)g * p.v_block + e] = vr[i];
        }
    }
}

// n consecutive floats of a row, 16 bytes at a time where they lie so
__device__ __forceinline__ float row_squares(const float *__restrict__ x, uint32_t n) {
    float m = 0.0f;
    if (n % 4 == 0 && (reinterpret_cast<uintptr_t>(x) & 15) == 0) {
#pragma unroll 4
        for (uint32_t i = threadIdx.x; i < n / 4; i += kThreads) {
            const float4 v = reinterpret_cast<const float4 *>(x)[i];
            m = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, m))));
        }
    } else {
        for (uint32_t i = threadIdx.x; i < n; i += kThreads) m = fmaf(x[i], x[i], m);
    }
    return m;
}

// Four lanes share a key; REP query heads of the kv head at a time (blockIdx.y = kv head and which of its head groups).
// FRESH (a few new tokens): the queries and the new keys are normed here, from the projections as they are, and a token's
// own workgroups of the last segment write its key and value rows into the cache; the cache is not read at new positions.
template <int REP, int VW, bool FRESH>
__global__ __launch_bounds__(kThreads) void attention_scores_kernel(const AttentionPlan p, const float *__restrict__ q, const uint32_t row0, const uint32_t nseg,
                                                                    float *__restrict__ scores, float2 *__restrict__ stats) {
    extern __shared__ float lds[]; // [REP][dim] queries, [REP][kSeg] scores, FRESH: [S][dim] new keys
    __shared__ float red[kWaves];
    const uint32_t rep = p.heads / p.kv_heads, groups = (rep + REP - 1) / REP;
    const uint32_t g = blockIdx.y / groups, h0 = g * rep + (blockIdx.y - g * groups) * REP, nh = min((uint32_t)REP, (g + 1) * rep - h0);
    const uint32_t r = row0 + blockIdx.z, b = r / p.S, s = r - b * p.S, seg = blockIdx.x;
    float *sc = lds + REP * p.dim, *fresh = sc + REP * kSeg;
    uint32_t lo, hi;
    visible(p, s, &lo, &hi);
    const uint32_t j0 = lo + seg * kSeg;
    if constexpr (FRESH) {
        const uint32_t nq = p.heads * p.dim, nk = p.kv_heads * p.dim;
        const float *qr = p.q.p + (int64_t)r * p.q.pitch;
        float f = p.scale;
        if (p.temp_every) f *= 1.0f + p.temp_coef * logf((float)((p.position + s + 1) / p.temp_every + 1));
        const float rms = p.q_norm ? 1.0f / sqrtf(block_sum(row_squares(qr, nq), red) / (float)nq + p.eps) : 1.0f;
        for (uint32_t i = threadIdx.x; i < REP * p.dim; i += kThreads) {
            const uint32_t h = i / p.dim, e = h0 * p.dim + i;
            float v = 0.0f;
            if (h < nh) v = p.q_norm ? qr[e] * rms * p.q_norm[e] : qr[e];
            lds[i] = v * f;
        }
        for (uint32_t t = 0; t <= s; t++) { // the new keys among this workgroup's
            const uint32_t j = p.cached + t;
            if (j < j0 || j >= j0 + kSeg) continue;
            const float *kr = p.k.p + ((int64_t)b * p.S + t) * p.k.pitch;
            const float fk = p.k_norm ? 1.0f / sqrtf(block_sum(row_squares(kr, nk), red) / (float)nk + p.eps) : 1.0f;
            float *kc = p.keys + ((int64_t)b * p.kv_heads + g) * p.k_block + (int64_t)j * p.dim;
            for (uint32_t d = threadIdx.x; d < p.dim; d += kThreads) {
                const float v = p.k_norm ? kr[g * p.dim + d] * fk * p.k_norm[g * p.dim + d] : kr[g * p.dim + d];
                fresh[t * p.dim + d] = v;
                if (t == s && h0 == g * rep) kc[d] = v;
            }
            if (t == s && h0 == g * rep)
                for (uint32_t d = threadIdx.x; d < p.vdim; d += kThreads)
                    p.values[((int64_t)b * p.kv_heads + g) * p.v_block + (int64_t)j * p.vdim + d] = p.v.p[(int64_t)r * p.v.pitch + g * p.vdim + d];
        }
    } else {
        for (uint32_t i = threadIdx.x; i < REP * p.dim; i += kThreads) {
            const uint32_t h = i / p.dim, d = i - h * p.dim;
            lds[i] = h < nh ? q[((int64_t)r * p.heads + h0 + h) * p.dim + d] : 0.0f;
        }
    }
    __syncthreads();
    const float *K = p.keys + ((int64_t)b * p.kv_heads + g) * p.k_block;
    const uint32_t sub = threadIdx.x & 3, nd = p.dim / VW;
    for (uint32_t key = threadIdx.x >> 2; key < kSeg; key += kThreads / 4) {
        const uint32_t j = j0 + key;
        float acc[REP] = {};
        if (j < hi) {
            auto walk = [&](const float *kp) {
#pragma unroll 4
                for (uint32_t i = sub; i < nd; i += 4) {
                    float kv[VW];
                    if constexpr (VW == 4) {
                        const float4 t = *reinterpret_cast<const float4 *>(kp + 4 * i);
                        kv[0] = t.x, kv[1] = t.y, kv[2] = t.z, kv[3] = t.w;
                    } else {
                        kv[0] = kp[i];
                    }
#pragma unroll
                    for (int h = 0; h < REP; h++)
#pragma unroll
                        for (int e = 0; e < VW; e++) acc[h] = fmaf(kv[e], lds[h * p.dim + VW * i + e], acc[h]);
                }
            };
            if (FRESH && j >= p.cached) walk(fresh + (j - p.cached) * p.dim);
            else walk(K + (int64_t)j * p.dim);
        }
#pragma unroll
        for (int h = 0; h < REP; h++) {
            float v = acc[h];
            v += __shfl_xor(v, 1, 64);
            v += __shfl_xor(v, 2, 64);
            if (sub == 0) {
                if (p.bias) v -= slope_of(h0 + h, p.heads) * (float)(int)(p.cached + s - j);
                sc[h * kSeg + key] = j < hi ? v : -INFINITY;
            }
        }
    }
    __syncthreads();
    const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    for (uint32_t h = wave; h < nh; h += kWaves) {
        const float a = sc[h * kSeg + lane], c = sc[h * kSeg + 64 + lane];
        float m = fmaxf(a, c);
#pragma unroll
        for (int d = 32; d > 0; d >>= 1) m = fmaxf(m, __shfl_xor(m, d, 64));
        const float l = m == -INFINITY ? 0.0f : wave_sum(expf(a - m) + expf(c - m));
        const int64_t head = (int64_t)blockIdx.z * p.heads + h0 + h;
        float *o = scores + (head * nseg + seg) * kSeg;
        o[lane] = a;
        o[64 + lane] = c;
        if (lane == 0) stats[head * nseg + seg] = make_float2(m, l);
    }
}

// LDS of the mixing kernel, in floats: with H' all heads when they are mixed, else the heads of a workgroup.
// [H'] maxima, [REP][H'] mixing factors over the sums, [H'][kSeg] exponentials, [REP][kSeg] weights, [REP][VW][256] results
__host__ __device__ constexpr uint32_t mix_floats(uint32_t rep, uint32_t slots, uint32_t vw) {
    return slots + rep * slots + slots * kSeg + rep * kSeg + rep * vw * kThreads;
}

template <int REP, int VW>
__global__ __launch_bounds__(kThreads) void attention_mix_kernel(const AttentionPlan p, const uint32_t row0, const uint32_t nseg, const float *__restrict__ scores,
                                                                 const float2 *__restrict__ stats, float *__restrict__ dst, const bool partial) {
    extern __shared__ float lds[];
    const uint32_t rep = p.heads / p.kv_heads, groups = (rep + REP - 1) / REP;
    const uint32_t g = blockIdx.y / groups, h0 = g * rep + (blockIdx.y - g * groups) * REP, nh = min((uint32_t)REP, (g + 1) * rep - h0);
    const uint32_t r = row0 + blockIdx.z, b = r / p.S, s = r - b * p.S, seg = blockIdx.x;
    const uint32_t first = p.talk ? 0 : h0, nm = p.talk ? p.heads : nh, slots = p.talk ? p.heads : REP;
    float *mx = lds, *tm = mx + slots, *ex = tm + REP * slots, *wt = ex + slots * kSeg, *red = wt + REP * kSeg;
    uint32_t lo, hi;
    visible(p, s, &lo, &hi);
    const uint32_t j0 = lo + seg * kSeg, keys = j0 < hi ? min(kSeg, hi - j0) : 0;
    const float *Vp = p.values + ((int64_t)b * p.kv_heads + g) * p.v_block + (int64_t)min(j0, hi - 1) * p.vdim;
    uint32_t lanes = 1; // lanes side by side along vdim; the others take keys in turn
    while (lanes < kThreads && lanes * VW < p.vdim) lanes *= 2;
    const uint32_t across = threadIdx.x & (lanes - 1), turn = threadIdx.x / lanes, turns = kThreads / lanes;
    // the values of the first columns are asked for before the weights are known
    constexpr int AHEAD = 16;
    float v[AHEAD][VW];
    auto load = [&](uint32_t d, uint32_t k, float(&t)[VW]) {
        // (clamped, not tested: what is not there is not used)
        const float *x = Vp + (int64_t)min(k, max(keys, 1u) - 1) * p.vdim + min(d, p.vdim - VW);
        if constexpr (VW == 4) {
            const float4 f = *reinterpret_cast<const float4 *>(x);
            t[0] = f.x, t[1] = f.y, t[2] = f.z, t[3] = f.w;
        } else {
            t[0] = *x;
        }
    };
#pragma unroll
    for (int i = 0; i < AHEAD; i++) load(across * VW, turn + i * turns, v[i]);
    const uint32_t key = threadIdx.x % kSeg; // two threads share a key's column of scores
    for (uint32_t h = threadIdx.x / kSeg; h < nm; h += kThreads / kSeg) ex[h * kSeg + key] = scores[(((int64_t)blockIdx.z * p.heads + first + h) * nseg + seg) * kSeg + key];
    for (uint32_t h = threadIdx.x; h < nm; h += kThreads) {
        const float2 *st = stats + ((int64_t)blockIdx.z * p.heads + first + h) * nseg;
        float m = p.zero_sink ? 0.0f : -INFINITY, l = p.zero_sink ? 1.0f : 0.0f;
#pragma unroll 4
        for (uint32_t i = 0; i < nseg; i++) { // the running pair: one walk along the segments
            const float2 t = st[i];
            const float up = fmaxf(m, t.x);
            if (t.y > 0.0f) l = (m == -INFINITY ? 0.0f : l * expf(m - up)) + t.y * expf(t.x - up);
            m = up;
        }
        mx[h] = m;
        for (uint32_t o = 0; o < REP; o++) {
            const float f = o >= nh ? 0.0f : p.talk ? p.talk[(int64_t)(h0 + o) * p.heads + h] : (o == h ? 1.0f : 0.0f);
            tm[o * slots + h] = f / l;
        }
    }
    __syncthreads();
    for (uint32_t h = threadIdx.x / kSeg; h < nm; h += kThreads / kSeg) ex[h * kSeg + key] = expf(ex[h * kSeg + key] - mx[h]); // (beyond the last key: 0)
    __syncthreads();
    for (uint32_t o = threadIdx.x / kSeg; o < REP; o += kThreads / kSeg) {
        float w = 0.0f;
#pragma unroll 4
        for (uint32_t h = 0; h < nm; h++) w = fmaf(tm[o * slots + h], ex[h * kSeg + key], w);
        wt[o * kSeg + key] = w;
    }
    __syncthreads();
    for (uint32_t d0 = 0; d0 < p.vdim; d0 += lanes * VW) {
        const uint32_t d = d0 + across * VW;
        float acc[REP][VW] = {};
        for (uint32_t k0 = turn; k0 < keys; k0 += AHEAD * turns) {
            if (d0 > 0 || k0 > turn)
#pragma unroll
                for (int i = 0; i < AHEAD; i++) load(d, k0 + i * turns, v[i]);
#pragma unroll
            for (int i = 0; i < AHEAD; i++) {
                const uint32_t k = k0 + i * turns;
                if (k < keys)
#pragma unroll
                    for (int o = 0; o < REP; o++) {
                        const float w = wt[o * kSeg + k];
#pragma unroll
                        for (int e = 0; e < VW; e++) acc[o][e] = fmaf(w, v[i][e], acc[o][e]);
                    }
            }
        }
#pragma unroll
        for (int o = 0; o < REP; o++)
#pragma unroll
            for (int e = 0; e < VW; e++) red[(o * VW + e) * kThreads + threadIdx.x] = acc[o][e];
        __syncthreads();
        const uint32_t cols = min(lanes * VW, p.vdim - d0);
        for (uint32_t i = threadIdx.x; i < nh * cols; i += kThreads) {
            const uint32_t o = i / cols, c = i - o * cols, h = h0 + o;
            float sum = 0.0f;
#pragma unroll 4
            for (uint32_t t = 0; t < turns; t++) sum += red[(o * VW + c % VW) * kThreads + t * lanes + c / VW];
            float *out = partial ? dst + (((int64_t)blockIdx.z * nseg + seg) * p.heads + h) * p.vdim : dst + ((int64_t)r * p.heads + h) * p.vdim;
            out[d0 + c] = sum;
        }
        __syncthreads();
    }
}

__global__ __launch_bounds__(kThreads) void attention_sum_kernel(const float *__restrict__ parts, const uint32_t nseg, const uint32_t n, float *__restrict__ out) {
    const uint32_t i = blockIdx.x * kThreads + threadIdx.x;
    if (i >= n) return;
    const float *p = parts + (int64_t)blockIdx.y * nseg * n + i;
    float s = 0.0f;
    for (uint32_t k = 0; k < nseg; k++) s += p[(int64_t)k * n];
    out[(int64_t)blockIdx.y * n + i] = s;
}

int launched(const char *what) {
    const hipError_t e = hipGetLastError();
    return e == hipSuccess ? CG_OK : hip_fail(e, what);
}

constexpr size_t kMaxLds = 128 << 10;
template <class F> int allow_lds(F *kernel, size_t bytes) {
    if (bytes > kMaxLds) return fail(CG_ERR_UNSUPPORTED, "block_attention: heads or sizes beyond what the kernels hold");
    if (bytes <= (64 << 10)) return CG_OK;
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kMaxLds);
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

template <int REP, int SVW, int MVW>
int rows_kernels(cg_backend *be, const AttentionPlan &p, const float *q, uint32_t row0, uint32_t rows, uint32_t nseg, float *scores, float2 *stats, float *parts) {
    const uint32_t rep = p.heads / p.kv_heads, groups = (rep + REP - 1) / REP, slots = p.talk ? p.heads : REP;
    const bool fresh = !q; // a few new tokens, not prepared
    const size_t lds1 = ((size_t)REP * p.dim + REP * kSeg + (fresh ? p.S * p.dim : 0)) * 4;
    const size_t lds2 = (size_t)mix_floats(REP, slots, MVW) * 4;
    if (int rc = fresh ? allow_lds(attention_scores_kernel<REP, SVW, true>, lds1) : allow_lds(attention_scores_kernel<REP, SVW, false>, lds1)) return rc;
    if (!p.mix_scores)
        if (int rc = allow_lds(attention_mix_kernel<REP, MVW>, lds2)) return rc;
    const dim3 grid(nseg, p.kv_heads * groups, rows);
    if (fresh) hipLaunchKernelGGL((attention_scores_kernel<REP, SVW, true>), grid, dim3(kThreads), lds1, be->stream, p, q, row0, nseg, scores, stats);
    else hipLaunchKernelGGL((attention_scores_kernel<REP, SVW, false>), grid, dim3(kThreads), lds1, be->stream, p, q, row0, nseg, scores, stats);
    if (p.mix_scores) return launch_mixed_rows(be, p, row0, rows, nseg, scores, parts, reinterpret_cast<float2 *>(parts + (size_t)rows * nseg * p.heads * p.vdim));
    hipLaunchKernelGGL((attention_mix_kernel<REP, MVW>), grid, dim3(kThreads), lds2, be->stream, p, row0, nseg, scores, stats, nseg > 1 ? parts : p.out, nseg > 1);
    if (nseg > 1) {
        const uint32_t n = p.heads * p.vdim;
        hipLaunchKernelGGL(attention_sum_kernel, dim3((n + kThreads - 1) / kThreads, rows), dim3(kThreads), 0, be->stream, parts, nseg, n,
                           p.out + (int64_t)row0 * n);
    }
    return launched("block_attention");
}

template <int REP>
int rows_kernels(cg_backend *be, const AttentionPlan &p, const float *q, uint32_t row0, uint32_t rows, uint32_t nseg, float *scores, float2 *stats, float *parts) {
    const bool dv = p.dim % 4 == 0, vv = p.vdim % 4 == 0; // (cache rows begin at multiples of their length: 16-byte loads then)
    if (dv && vv) return rows_kernels<REP, 4, 4>(be, p, q, row0, rows, nseg, scores, stats, parts);
    if (dv) return rows_kernels<REP, 4, 1>(be, p, q, row0, rows, nseg, scores, stats, parts);
    if (vv) return rows_kernels<REP, 1, 4>(be, p, q, row0, rows, nseg, scores, stats, parts);
    return rows_kernels<REP, 1, 1>(be, p, q, row0, rows, nseg, scores, stats, parts);
}

} // namespace

// The tables of a plan's rotation, for the positions before `end`: made when a model first asks for them, the coarse one in
// powers of two.
static int rotation_tables(cg_backend *be, AttentionPlan &p, uint64_t end) {
    const uint32_t pairs = p.rot_dims / 2;
    RotTable *t = nullptr;
    for (RotTable &r : be->rot_tables)
        if (r.dims == p.rot_dims && r.log2_base == p.rot_log2) t = &r;
    auto fill = [&](uint32_t rows, uint32_t step, Buffer **out) {
        Buffer *b = new Buffer;
        b->be = be;
        b->elems = (int64_t)rows * pairs * 2;
        if (int rc = be->pool.alloc((size_t)b->elems * 4, &b->ptr, &b->cls)) {
            delete b;
            return rc;
        }
        hipLaunchKernelGGL(rotation_table_kernel, dim3((rows * pairs + kThreads - 1) / kThreads), dim3(kThreads), 0, be->stream, static_cast<float2 *>(b->ptr), rows, step,
                           p.rot_dims, p.rot_log2);
        *out = b;
        return launched("rotation_table");
    };
    const uint64_t need = (end + kRotFine - 1) / kRotFine;
    if (need > (1u << 24) / std::max(1u, pairs)) return fail(CG_ERR_UNSUPPORTED, "block_attention: a position beyond the rotation's tables");
    if (!t) {
        RotTable r{p.rot_dims, p.rot_log2, nullptr, nullptr, 0};
        if (int rc = fill(kRotFine, 1, &r.fine)) return rc;
        uint32_t n = 16;
        while (n < need) n *= 2;
        if (int rc = fill(n, kRotFine, &r.coarse)) {
            buffer_release(r.fine);
            return rc;
        }
        r.coarse_n = n;
        be->rot_tables.push_back(r);
        t = &be->rot_tables.back();
    } else if (need > t->coarse_n) {
        uint32_t n = t->coarse_n;
        while (n < need) n *= 2;
        Buffer *b = nullptr;
        if (int rc = fill(n, kRotFine, &b)) return rc;
        buffer_release(t->coarse); // (stream-ordered)
        t->coarse = b;
        t->coarse_n = n;
    }
    p.rot_fine = static_cast<const float2 *>(t->fine->ptr);
    p.rot_coarse = static_cast<const float2 *>(t->coarse->ptr);
    return CG_OK;
}

int launch_attention(cg_backend *be, const AttentionPlan &plan) {
    AttentionPlan p = plan;
    if (p.rot_dims)
        if (int rc = rotation_tables(be, p, p.position + p.S)) return rc;
    const uint32_t rows = p.B * p.S, all = p.cached + p.S;
    const bool turned = p.rot_dims || p.unit_heads, fresh = p.S <= kFewRows && p.dim <= 512 && !turned;
    const uint32_t most = p.window ? std::min(p.window, all) : all, nseg = (most + kSeg - 1) / kSeg, rep = p.heads / p.kv_heads;
    double pairs = 0.0; // visible (query, key) pairs
    for (uint32_t s = 0; s < p.S; s++) pairs += (double)std::min(p.window ? p.window : ~0u, p.cached + s + 1);
    ProfScope prof(be, CG_K_ATTENTION, pairs * p.B * p.heads * (2.0 * p.dim + 2.0 * p.vdim + (p.talk ? 2.0 * p.heads : 0.0)));
    if (p.mix_scores)
        if (int rc = launch_mixed_step(be, p); rc != kDeclined) return rc;
    Scratch qbuf(be);
    float *q = nullptr;
    if (!fresh) {
        if (int rc = qbuf.get((size_t)rows * p.heads * p.dim * 4)) return rc;
        q = static_cast<float *>(qbuf.p);
        auto aligned = [](const Rows &x) { return x.pitch % 4 == 0 && (reinterpret_cast<uintptr_t>(x.p) & 15) == 0; };
        const bool pieces = turned && !p.q_norm && !p.k_norm && p.dim % 4 == 0 && p.dim <= 256 && aligned(p.q) && aligned(p.k);
        if (pieces && p.dim <= 32) hipLaunchKernelGGL((attention_turn_heads_kernel<8>), dim3(rows), dim3(kThreads), 0, be->stream, p, q);
        else if (pieces && p.dim <= 64) hipLaunchKernelGGL((attention_turn_heads_kernel<16>), dim3(rows), dim3(kThreads), 0, be->stream, p, q);
        else if (pieces && p.dim <= 128) hipLaunchKernelGGL((attention_turn_heads_kernel<32>), dim3(rows), dim3(kThreads), 0, be->stream, p, q);
        else if (pieces) hipLaunchKernelGGL((attention_turn_heads_kernel<64>), dim3(rows), dim3(kThreads), 0, be->stream, p, q);
        else if (turned) hipLaunchKernelGGL(attention_turn_kernel, dim3(rows), dim3(kThreads), (size_t)(p.rot_dims / 2) * sizeof(float2), be->stream, p, q);
        else hipLaunchKernelGGL(attention_prepare_kernel, dim3(rows), dim3(kThreads), 0, be->stream, p, q);
        if (int rc = launched("attention_prepare")) return rc;
        if (int rc = p.mix_scores ? launch_mixed_tiles(be, p, q) : launch_attention_tiles(be, p, q); rc != kDeclined) return rc;
    }
    // rows in parts that keep the scores within 64 MB
    const size_t per_row = (size_t)p.heads * nseg * (kSeg * 4 + sizeof(float2)) + (nseg > 1 || p.mix_scores ? (size_t)nseg * p.heads * (p.vdim * 4 + (p.mix_scores ? sizeof(float2) : 0)) : 0);
    const uint32_t part = (uint32_t)std::max<size_t>(1, std::min<size_t>(std::min<size_t>(rows, 65535), (64u << 20) / per_row));
    Scratch mem(be);
    if (int rc = mem.get((size_t)part * per_row)) return rc;
    float *scores = static_cast<float *>(mem.p);
    float2 *stats = reinterpret_cast<float2 *>(scores + (size_t)part * p.heads * nseg * kSeg);
    float *parts = reinterpret_cast<float *>(stats + (size_t)part * p.heads * nseg);
    for (uint32_t r0 = 0; r0 < rows; r0 += part) {
        const uint32_t n = std::min(part, rows - r0);
        int rc = rep <= 1   ? rows_kernels<1>(be, p, q, r0, n, nseg, scores, stats, parts)
                 : rep <= 2 ? rows_kernels<2>(be, p, q, r0, n, nseg, scores, stats, parts)
                 : rep <= 4 ? rows_kernels<4>(be, p, q, r0, n, nseg, scores, stats, parts)
                            : rows_kernels<8>(be, p, q, r0, n, nseg, scores, stats, parts);
        if (rc) return rc;
    }
    return CG_OK;
}

} // namespace cg
