// The delta rule with a state that decays channel by channel (cg_block_channel_delta).
//
// A few new tokens (a decode step): delta_step_kernel, a workgroup per (sequence, head) that does everything from the
// convolutions to the gated norm, the state in registers from the first token to the last.
//
// More: chunks of 16 tokens.  With G_t the sum of the logarithms of the decays from the chunk's start to token t (per key
// channel), S_0 the state before the chunk and S the one behind it,
//     M[t, s] = sum_d k_t k_s exp(G_t - G_s)  (s < t),   A[t, s] = sum_d q_t k_s exp(G_t - G_s)  (s <= t),
//     T = (I + diag(beta) M)^-1 diag(beta),              U = T V - (T (k exp G)) S_0 = U' - W S_0,
//     O = (q exp G) S_0 + A U,                           S = exp(G_15) S_0 + (k exp(G_15 - G))^T U.
// Every exponent is of a difference that is not positive, so no decay, however fast, overflows.
//   delta_chunk_kernel   everything that does not need S_0, a workgroup per (chunk, head): convolutions, norms, decays, M, A,
//                        T, W, U' and the scaled queries and keys
//   delta_scan_kernel    the walk along the chunks on v_mfma_f32_16x16x4, 16 columns of the state per wave, its rows cut over
//                        four waves
//   delta_finish_kernel  a wave per (token, head): the norm over the head's values and the gate
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
// on the hardware's exp2, log2 and reciprocal (about one unit in the last place each)
__device__ __forceinline__ float sigmoid(float z) { return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(z * -1.44269504088896341f)); }
// max(z, 0) + ln(1 + e^-|z|), by its series where 1 + e^-|z| would lose what a slow decay lives on
__device__ __forceinline__ float softplus(float z) {
    const float t = __builtin_amdgcn_exp2f(-fabsf(z) * 1.44269504088896341f);
    const float l = t < 0.01f ? t * fmaf(t, fmaf(t, 0.33333333f, -0.5f), 1.0f) : __builtin_amdgcn_logf(1.0f + t) * 0.69314718055994531f;
    return fmaxf(z, 0.0f) + l;
}

// Channel c of the three projections side by side: where its column of tokens begins (at sequence b, token 0), and its taps.
// (Values are selected, not references: a reference into the arguments would have them fetched lane by lane.)
struct Channel {
    const float *x, *taps;
    int64_t pitch;
};
__device__ __forceinline__ Channel channel(const DeltaPlan &p, uint32_t b, uint32_t c) {
    const uint32_t kc = p.kv_heads * p.dim;
    const bool is_q = c < kc, is_k = c < 2 * kc;
    const uint32_t e = is_q ? c : is_k ? c - kc : c - 2 * kc;
    const float *x = is_q ? p.q.p : is_k ? p.k.p : p.v.p, *w = is_q ? p.conv_q : is_k ? p.conv_k : p.conv_v;
    const int64_t pitch = is_q ? p.q.pitch : is_k ? p.k.pitch : p.v.pitch;
    return {x + (int64_t)b * p.S * pitch + e, w + (int64_t)e * p.taps, pitch};
}
// its input at time t (t < 0: what the state kept)
__device__ __forceinline__ float conv_input(const DeltaPlan &p, const Channel &ch, uint32_t b, int t, uint32_t c) {
    if (t >= 0) return ch.x[(int64_t)t * ch.pitch];
    const uint32_t C = 2 * p.kv_heads * p.dim + p.heads * p.vdim;
    return p.conv_state ? p.conv_state[((int64_t)b * (p.taps - 1) + (t + (int)p.taps - 1)) * C + c] : 0.0f;
}
__device__ __forceinline__ float conv_silu(const DeltaPlan &p, uint32_t b, int t, uint32_t c) {
    const Channel ch = channel(p, b, c);
    float s = 0.0f;
    for (uint32_t i = 0; i < p.taps; i++) s = fmaf(conv_input(p, ch, b, t - (int)(p.taps - 1 - i), c), ch.taps[i], s);
    return s * sigmoid(s);
}

constexpr float kLog2e = 1.44269504088896341f;
constexpr uint32_t kChunk = 16;
__device__ __forceinline__ float exp2_of(float x) { return __builtin_amdgcn_exp2f(x); } // (x <= 0)

// log2 of the decay of key channel d of head h
__device__ __forceinline__ float log2_decay(const DeltaPlan &p, float a, uint32_t h, uint32_t d) {
    return -expf(p.a_log[h]) * softplus(a + p.dt_bias[h * p.dim + d]) * kLog2e;
}

// The last taps - 1 inputs of head h's channels (of its q and k channels if it is the first head that uses them).
__device__ void keep_inputs(const DeltaPlan &p, uint32_t b, uint32_t h) {
    const uint32_t kc = p.kv_heads * p.dim, C = 2 * kc + p.heads * p.vdim, past = p.taps - 1, rep = p.heads / p.kv_heads;
    const uint32_t nq = h % rep == 0 ? p.dim : 0, n = 2 * nq + p.vdim;
    for (uint32_t i = threadIdx.x; i < past * n; i += blockDim.x) {
        const uint32_t j = i / n, e = i - j * n;
        const uint32_t c = e < nq ? (h / rep) * p.dim + e : e < 2 * nq ? kc + (h / rep) * p.dim + (e - nq) : 2 * kc + h * p.vdim + (e - 2 * nq);
        p.conv_out[((int64_t)b * past + j) * C + c] = conv_input(p, channel(p, b, c), b, (int)(p.S + j) - (int)past, c);
    }
}

// What delta_chunk_kernel leaves per (sequence, head, chunk): W, the queries times exp(G) [16][DP] each, the keys times
// exp(G_15 - G) as [DP][16], A [16][16], exp(G_15) [DP], with DP the key channels rounded up to a multiple of 64 (zeros
// there); and U' [16][vdim].
struct ChunkArrays {
    float *mats, *u;
    uint32_t dp, chunks; // chunks of a sequence in this part of the tokens
    uint32_t first;      // first token of this part
};
__device__ __host__ constexpr uint32_t chunk_floats(uint32_t dp) { return 48 * dp + 256 + dp; }

// Outputs of the convolution of channel c (of 16 tokens from t0; n of them are there), silu applied.  TAPS 0: any count.
template <int TAPS> __device__ __forceinline__ void conv_chunk(const DeltaPlan &p, uint32_t b, uint32_t t0, uint32_t n, uint32_t c, float (&y)[kChunk]) {
    if constexpr (TAPS > 0) {
        const Channel ch = channel(p, b, c);
        const float *x = ch.x + (int64_t)t0 * ch.pitch;
        float in[kChunk + TAPS - 1], wt[TAPS];
#pragma unroll
        for (uint32_t t = 0; t < kChunk; t++) in[t + TAPS - 1] = x[(int64_t)min(t, n - 1) * ch.pitch]; // (clamped, not tested: no load waits)
#pragma unroll
        for (int i = 0; i < TAPS; i++) wt[i] = ch.taps[i];
        if (t0 >= TAPS - 1) {
#pragma unroll
            for (int i = 0; i < TAPS - 1; i++) in[i] = x[(int64_t)(i - (TAPS - 1)) * ch.pitch];
        } else {
#pragma unroll
            for (int i = 0; i < TAPS - 1; i++) in[i] = conv_input(p, ch, b, (int)t0 + i - (TAPS - 1), c);
        }
#pragma unroll
        for (uint32_t t = 0; t < kChunk; t++) {
            float s = 0.0f;
#pragma unroll
            for (int i = 0; i < TAPS; i++) s = fmaf(in[t + i], wt[i], s);
            y[t] = t < n ? s * sigmoid(s) : 0.0f;
        }
    } else {
#pragma unroll
        for (uint32_t t = 0; t < kChunk; t++) y[t] = t < n ? conv_silu(p, b, (int)(t0 + t), c) : 0.0f;
    }
}

template <int TAPS> __global__ __launch_bounds__(kThreads, 2) void delta_chunk_kernel(const DeltaPlan p, const ChunkArrays o, const float *__restrict__ decay) {
    extern __shared__ float lds[]; // q, k, G: [16][pitch] each
    __shared__ float beta[kChunk], lower[kChunk][kChunk + 4], tb[kChunk][kChunk + 4]; // tb[s][t] = T[t][s]
    const uint32_t chunk = blockIdx.x, h = blockIdx.y, b = blockIdx.z, rep = p.heads / p.kv_heads, g = h / rep;
    const uint32_t t0 = o.first + chunk * kChunk, n = min(kChunk, p.S - t0), D = p.dim, dp = o.dp, pitch = dp + 4, kc = p.kv_heads * D;
    float *q = lds, *k = q + kChunk * pitch, *G = k + kChunk * pitch;
    const uint32_t tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    if (tid < kChunk) beta[tid] = tid < n ? sigmoid(p.beta.p[((int64_t)b * p.S + t0 + tid) * p.beta.pitch + h]) : 0.0f;
    for (uint32_t u = tid; u < 3 * dp; u += kThreads) {
        const uint32_t which = u / dp, d = u - which * dp;
        float y[kChunk];
        if (d >= D) {
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t++) y[t] = 0.0f;
        } else if (which < 2) {
            conv_chunk<TAPS>(p, b, t0, n, which * kc + g * D + d, y);
        } else {
            const float *a = decay + ((int64_t)b * p.S + t0) * p.heads * D + h * D + d;
            const float rate = -expf(p.a_log[h]) * kLog2e, bias = p.dt_bias[h * D + d];
            float sum = 0.0f;
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t++) y[t] = a[(int64_t)min(t, n - 1) * p.heads * D];
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t++) {
                sum += t < n ? rate * softplus(y[t] + bias) : 0.0f;
                y[t] = sum;
            }
        }
#pragma unroll
        for (uint32_t t = 0; t < kChunk; t++) lds[(which * kChunk + t) * pitch + d] = y[t];
    }
    if (t0 == 0) keep_inputs(p, b, h);
    __syncthreads();
    for (uint32_t u = wave; u < 2 * kChunk; u += kWaves) { // the unit vectors: rows of q, then of k
        float *row = lds + u * pitch, ss = 0.0f;
        for (uint32_t d = lane; d < dp; d += 64) ss = fmaf(row[d], row[d], ss);
        float f = 1.0f / sqrtf(wave_sum(ss) + 1e-6f);
        if (u < kChunk) f *= 1.0f / sqrtf((float)D);
        for (uint32_t d = lane; d < dp; d += 64) row[d] *= f;
    }
    __syncthreads();
    float *mats = o.mats + (((int64_t)b * p.heads + h) * o.chunks + chunk) * chunk_floats(dp);
    float *W = mats, *Q = W + kChunk * dp, *K = Q + kChunk * dp, *A = K + kChunk * dp, *E = A + kChunk * kChunk;
    // the 120 pairs s < t, two lanes each (the key channels' quads in turn); the other 16 threads take A's diagonal
    if (tid < kChunk * (kChunk - 1)) {
        const uint32_t pair = tid >> 1;
        uint32_t t = (uint32_t)((1.0f + sqrtf(8.0f * (float)pair + 1.0f)) * 0.5f); // row of the pair-th entry below the diagonal
        t -= t * (t - 1) / 2 > pair ? 1 : 0;
        t += t * (t + 1) / 2 <= pair ? 1 : 0;
        const uint32_t s = pair - t * (t - 1) / 2;
        float m = 0.0f, a = 0.0f;
        for (uint32_t d = (tid & 1) * 4; d < dp; d += 8) { // (zeros behind the last channel)
            const float4 gt = *reinterpret_cast<const float4 *>(G + t * pitch + d), gs = *reinterpret_cast<const float4 *>(G + s * pitch + d);
            const float4 kt = *reinterpret_cast<const float4 *>(k + t * pitch + d), qt = *reinterpret_cast<const float4 *>(q + t * pitch + d);
            float4 ks = *reinterpret_cast<const float4 *>(k + s * pitch + d);
            ks.x *= exp2_of(gt.x - gs.x);
            ks.y *= exp2_of(gt.y - gs.y);
            ks.z *= exp2_of(gt.z - gs.z);
            ks.w *= exp2_of(gt.w - gs.w);
            m = fmaf(kt.x, ks.x, fmaf(kt.y, ks.y, fmaf(kt.z, ks.z, fmaf(kt.w, ks.w, m))));
            a = fmaf(qt.x, ks.x, fmaf(qt.y, ks.y, fmaf(qt.z, ks.z, fmaf(qt.w, ks.w, a))));
        }
        m += __shfl_xor(m, 1, 64);
        a += __shfl_xor(a, 1, 64);
        if ((tid & 1) == 0) {
            lower[t][s] = beta[t] * m;
            A[t * kChunk + s] = a;
            A[s * kChunk + t] = 0.0f;
        }
    } else {
        const uint32_t t = tid - kChunk * (kChunk - 1);
        float a = 0.0f;
        for (uint32_t d = 0; d < dp; d += 4) {
            const float4 kt = *reinterpret_cast<const float4 *>(k + t * pitch + d), qt = *reinterpret_cast<const float4 *>(q + t * pitch + d);
            a = fmaf(qt.x, kt.x, fmaf(qt.y, kt.y, fmaf(qt.z, kt.z, fmaf(qt.w, kt.w, a))));
        }
        A[t * kChunk + t] = a;
    }
    __syncthreads();
    if (wave == 0) { // T: forward substitution, a lane per column
        if (lane < kChunk) {
            float x[kChunk];
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t++) {
                float v = t == lane ? 1.0f : 0.0f;
#pragma unroll
                for (uint32_t s = 0; s < t; s++) v = fmaf(-lower[t][s], x[s], v);
                x[t] = v;
            }
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t++) tb[lane][t] = x[t] * beta[lane];
        }
    } else {
        for (uint32_t d = tid - 64; d < dp; d += kThreads - 64) {
            const float last = G[(kChunk - 1) * pitch + d];
            E[d] = d < D ? exp2_of(last) : 0.0f;
            float kt[kChunk];
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t++) {
                const float gt = G[t * pitch + d];
                Q[t * dp + d] = q[t * pitch + d] * exp2_of(gt);
                kt[t] = k[t * pitch + d] * exp2_of(last - gt);
            }
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t += 4) *reinterpret_cast<float4 *>(K + d * kChunk + t) = make_float4(kt[t], kt[t + 1], kt[t + 2], kt[t + 3]);
        }
    }
    __syncthreads();
    float *U = o.u + (((int64_t)b * p.heads + h) * o.chunks + chunk) * kChunk * p.vdim;
    for (uint32_t u = tid; u < dp + p.vdim; u += kThreads) { // columns of W, then of U'
        float x[kChunk], y[kChunk];
        if (u < dp) {
#pragma unroll
            for (uint32_t s = 0; s < kChunk; s++) x[s] = k[s * pitch + u] * exp2_of(G[s * pitch + u]);
        } else {
            conv_chunk<TAPS>(p, b, t0, n, 2 * kc + h * p.vdim + (u - dp), x);
        }
#pragma unroll
        for (uint32_t t = 0; t < kChunk; t++) y[t] = 0.0f;
#pragma unroll
        for (uint32_t s = 0; s < kChunk; s++) {
#pragma unroll
            for (uint32_t t4 = s / 4 * 4; t4 < kChunk; t4 += 4) {
                const float4 f = *reinterpret_cast<const float4 *>(&tb[s][t4]);
                y[t4] = fmaf(f.x, x[s], y[t4]);
                y[t4 + 1] = fmaf(f.y, x[s], y[t4 + 1]);
                y[t4 + 2] = fmaf(f.z, x[s], y[t4 + 2]);
                y[t4 + 3] = fmaf(f.w, x[s], y[t4 + 3]);
            }
        }
        if (u < dp) {
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t++) W[t * dp + u] = y[t];
        } else {
#pragma unroll
            for (uint32_t t = 0; t < kChunk; t++) U[t * p.vdim + (u - dp)] = y[t];
        }
    }
}

typedef float f32x4 __attribute__((ext_vector_type(4)));
__device__ __forceinline__ f32x4 mfma(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// Floats of one chunk's matrices in LDS, rows padded off each other's banks.
__device__ __host__ constexpr uint32_t chunk_lds_floats(uint32_t dp) { return 2 * kChunk * (dp + 4) + dp * (kChunk + 4) + kChunk * (kChunk + 4) + dp; }

// CT groups of four waves, each with 16 columns of the state; wave w of a group holds TPW row tiles of 16.  What a lane
// holds of a tile — rows 4 (lane / 16) + r of column lane % 16 — is both what the instruction leaves and what it takes as
// its second operand, so the state and U never change place.
template <int TPW, int CT>
__global__ __launch_bounds__(CT * 256) void delta_scan_kernel(const DeltaPlan p, const ChunkArrays in, const float *__restrict__ state, float *__restrict__ out) {
    constexpr uint32_t DP = 64 * TPW, PITCH = DP + 4, TP = kChunk + 4, kAll = chunk_floats(DP), kQuads = kAll / 4;
    constexpr uint32_t SLOTS = (kQuads + CT * 256 - 1) / (CT * 256);
    extern __shared__ float lds[]; // two chunks' matrices, then the partial products [CT][4 waves][2][64] float4
    constexpr uint32_t LW = 0, LQ = LW + kChunk * PITCH, LK = LQ + kChunk * PITCH, LA = LK + DP * TP, LE = LA + kChunk * TP, kOne = LE + DP;
    f32x4 *part = reinterpret_cast<f32x4 *>(lds + 2 * kOne);
    const uint32_t h = blockIdx.y, b = blockIdx.z, wave = threadIdx.x >> 6, lane = threadIdx.x & 63, li = lane & 15, lg = lane >> 4;
    const uint32_t ct = wave >> 2, ds = wave & 3, col = (blockIdx.x * CT + ct) * 16 + li, D = p.dim, V = p.vdim;
    const bool live = col < V;
    f32x4 S[TPW];
    const int64_t sb = ((int64_t)b * p.heads + h) * D * V;
#pragma unroll
    for (int i = 0; i < TPW; i++)
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const uint32_t d = (ds * TPW + i) * 16 + 4 * lg + r;
            S[i][r] = live && state && d < D ? state[sb + (int64_t)d * V + col] : 0.0f;
        }
    const f32x4 *mats = reinterpret_cast<const f32x4 *>(in.mats + ((int64_t)b * p.heads + h) * in.chunks * kAll);
    const float *us = in.u + ((int64_t)b * p.heads + h) * in.chunks * kChunk * V;
    uint32_t to[SLOTS]; // where this thread's quads of a chunk go in LDS
#pragma unroll
    for (uint32_t i = 0; i < SLOTS; i++) {
        const uint32_t e = (i * CT * 256 + threadIdx.x) * 4;
        if (e < 2 * kChunk * DP) to[i] = e / DP * PITCH + e % DP; // W and Q lie behind each other
        else if (e < 3 * kChunk * DP) to[i] = LK + (e - 2 * kChunk * DP) / kChunk * TP + e % kChunk;
        else if (e < 3 * kChunk * DP + kChunk * kChunk) to[i] = LA + (e - 3 * kChunk * DP) / kChunk * TP + e % kChunk;
        else to[i] = LE + (e - 3 * kChunk * DP - kChunk * kChunk);
    }
    f32x4 stage[SLOTS], un;
    auto ask = [&](uint32_t c) {
#pragma unroll
        for (uint32_t i = 0; i < SLOTS; i++) {
            const uint32_t e = i * CT * 256 + threadIdx.x;
            if (e < kQuads) stage[i] = mats[(int64_t)c * kQuads + e];
        }
#pragma unroll
        for (int r = 0; r < 4; r++) un[r] = live ? us[((int64_t)c * kChunk + 4 * lg + r) * V + col] : 0.0f;
    };
    auto put = [&](float *dst) {
#pragma unroll
        for (uint32_t i = 0; i < SLOTS; i++)
            if (i * CT * 256 + threadIdx.x < kQuads) *reinterpret_cast<f32x4 *>(dst + to[i]) = stage[i];
    };
    ask(0);
    put(lds);
    f32x4 U = un;
    __syncthreads();
    for (uint32_t c = 0; c < in.chunks; c++) {
        const float *m = lds + (c & 1) * kOne;
        const bool more = c + 1 < in.chunks;
        if (more) ask(c + 1);
        f32x4 w = {0.0f, 0.0f, 0.0f, 0.0f}, y = w;
#pragma unroll
        for (int i = 0; i < TPW; i++) {
            const uint32_t d = (ds * TPW + i) * 16 + 4 * lg;
            const f32x4 a = *reinterpret_cast<const f32x4 *>(m + LW + li * PITCH + d), q = *reinterpret_cast<const f32x4 *>(m + LQ + li * PITCH + d);
#pragma unroll
            for (int t = 0; t < 4; t++) {
                w = mfma(a[t], S[i][t], w);
                y = mfma(q[t], S[i][t], y);
            }
        }
        part[((ct * 4 + ds) * 2) * 64 + lane] = w;
        part[((ct * 4 + ds) * 2 + 1) * 64 + lane] = y;
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 4; i++) U -= part[((ct * 4 + i) * 2) * 64 + lane];
        if (ds == (c & 3)) { // the waves of a group take the output in turn
            y = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int i = 0; i < 4; i++) y += part[((ct * 4 + i) * 2 + 1) * 64 + lane];
            const f32x4 a = *reinterpret_cast<const f32x4 *>(m + LA + li * TP + 4 * lg);
#pragma unroll
            for (int t = 0; t < 4; t++) y = mfma(a[t], U[t], y);
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const uint32_t t = in.first + c * kChunk + 4 * lg + r;
                if (live && t < p.S) out[(((int64_t)b * p.S + t) * p.heads + h) * V + col] = y[r];
            }
        }
#pragma unroll
        for (int i = 0; i < TPW; i++) {
            const uint32_t tile = (ds * TPW + i) * 16;
            S[i] *= *reinterpret_cast<const f32x4 *>(m + LE + tile + 4 * lg);
            const f32x4 kt = *reinterpret_cast<const f32x4 *>(m + LK + (tile + li) * TP + 4 * lg);
#pragma unroll
            for (int t = 0; t < 4; t++) S[i] = mfma(kt[t], U[t], S[i]);
        }
        if (more) {
            put(lds + ((c + 1) & 1) * kOne);
            U = un;
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < TPW; i++)
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const uint32_t d = (ds * TPW + i) * 16 + 4 * lg + r;
            if (live && d < D) p.state_out[sb + (int64_t)d * V + col] = S[i][r];
        }
}

// ---- a few tokens ----------------------------------------------------------------------------------------------------
constexpr int kStepThreads = 512;

__device__ __forceinline__ float step_sum(float v, float *red) { // over the workgroup, for every thread
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = 0.0f;
#pragma unroll
    for (int i = 0; i < kStepThreads / 64; i++) s += red[i];
    return s;
}
// w[row, :] . x, four lanes of a quad together
__device__ __forceinline__ float quad_dot(const float *__restrict__ w, const float *__restrict__ x, uint32_t n, uint32_t sub) {
    float s = 0.0f;
    if (n % 4 == 0 && ((reinterpret_cast<uintptr_t>(w) | reinterpret_cast<uintptr_t>(x)) & 15) == 0) { // (the same for every lane)
        constexpr int AHEAD = 4;
        const uint32_t quads = n / 4;
        for (uint32_t i0 = sub; i0 < quads; i0 += 4 * AHEAD) {
            float4 a[AHEAD], c[AHEAD];
#pragma unroll
            for (int j = 0; j < AHEAD; j++) {
                a[j] = reinterpret_cast<const float4 *>(w)[min(i0 + 4 * j, quads - 1)];
                c[j] = reinterpret_cast<const float4 *>(x)[min(i0 + 4 * j, quads - 1)];
            }
#pragma unroll
            for (int j = 0; j < AHEAD; j++) {
                const float t = fmaf(a[j].x, c[j].x, fmaf(a[j].y, c[j].y, fmaf(a[j].z, c[j].z, a[j].w * c[j].w)));
                s += i0 + 4 * j < quads ? t : 0.0f;
            }
        }
    } else {
        for (uint32_t i = sub; i < n; i += 4) s = fmaf(w[i], x[i], s);
    }
    s += __shfl_xor(s, 1, 64);
    s += __shfl_xor(s, 2, 64);
    return s;
}

// conv_silu with the inputs and taps asked for together when there are TAPS of them
template <int TAPS> __device__ __forceinline__ float conv_step(const DeltaPlan &p, uint32_t b, int t, uint32_t c) {
    if constexpr (TAPS == 0) {
        return conv_silu(p, b, t, c);
    } else {
        const uint32_t C = 2 * p.kv_heads * p.dim + p.heads * p.vdim;
        const Channel ch = channel(p, b, c);
        const float *now = ch.x + (int64_t)t * ch.pitch;
        const float *kept = p.conv_state ? p.conv_state + ((int64_t)b * (TAPS - 1) + t + TAPS - 1) * C + c : now;
        const int64_t kept_pitch = p.conv_state ? C : 0;
        float x[TAPS], tap[TAPS], s = 0.0f;
#pragma unroll
        for (int i = 0; i < TAPS; i++) {
            const int back = TAPS - 1 - i; // tokens before t
            tap[i] = ch.taps[i];
            x[i] = *(back <= t ? now - (int64_t)back * ch.pitch : kept - (int64_t)back * kept_pitch); // (one load, whichever it is)
        }
#pragma unroll
        for (int i = 0; i < TAPS; i++) x[i] = TAPS - 1 - i <= t || p.conv_state ? x[i] : 0.0f;
#pragma unroll
        for (int i = 0; i < TAPS; i++) s = fmaf(x[i], tap[i], s);
        return s * sigmoid(s);
    }
}

// Thread (c, group) holds rows group, group + groups, ... (at most R) of column c of the head's state.
template <int R, int TAPS> __global__ __launch_bounds__(kStepThreads) void delta_step_kernel(const DeltaPlan p, const uint32_t lanes) {
    __shared__ float q[257], k[257], g[257], v[kStepThreads], gate[kStepThreads], part[kStepThreads], red[kStepThreads / 64];
    const uint32_t h = blockIdx.x, b = blockIdx.y, rep = p.heads / p.kv_heads, kh = h / rep, D = p.dim, V = p.vdim, kc = p.kv_heads * D;
    const uint32_t tid = threadIdx.x, c = tid & (lanes - 1), group = tid / lanes, groups = kStepThreads / lanes;
    const int64_t sb = ((int64_t)b * p.heads + h) * D * V;
    float S[R];
    if (p.state) { // (clamped, not tested: no load waits)
        const float *src = p.state + sb + min(c, V - 1);
#pragma unroll
        for (int i = 0; i < R; i++) S[i] = src[(int64_t)min(group + i * groups, D - 1) * V];
#pragma unroll
        for (int i = 0; i < R; i++) S[i] = group + i * groups < D ? S[i] : 0.0f;
    } else {
#pragma unroll
        for (int i = 0; i < R; i++) S[i] = 0.0f;
    }
    if (tid == 0) q[D] = k[D] = g[D] = 0.0f; // what the rows behind the last one read
    for (uint32_t t = 0; t < p.S; t++) {
        const int64_t r = (int64_t)b * p.S + t;
        float sq = 0.0f, sk = 0.0f;
        for (uint32_t u = tid; u < 2 * D + V; u += kStepThreads) {
            const bool is_q = u < D, is_k = !is_q && u < 2 * D;
            const uint32_t e = is_q ? u : is_k ? u - D : u - 2 * D;
            const float x = conv_step<TAPS>(p, b, (int)t, (is_q ? kh * D : is_k ? kc + kh * D : 2 * kc + h * V) + e);
            sq = is_q ? fmaf(x, x, sq) : sq;
            sk = is_k ? fmaf(x, x, sk) : sk;
            (is_q ? q : is_k ? k : v)[e] = x;
        }
        for (uint32_t u = tid / 4; u < D + V; u += kStepThreads / 4) { // the two factored projections
            const bool is_g = u < D;
            const uint32_t e = is_g ? u : u - D;
            const float a = quad_dot(is_g ? p.decay_w + ((int64_t)h * D + e) * p.decay_rank : p.gate_w + ((int64_t)h * V + e) * p.gate_rank,
                                     is_g ? p.decay.p + r * p.decay.pitch : p.gate.p + r * p.gate.pitch, is_g ? p.decay_rank : p.gate_rank, tid & 3);
            if ((tid & 3) == 0) {
                if (is_g) g[e] = exp2_of(log2_decay(p, a, h, e));
                else gate[e] = sigmoid(a);
            }
        }
        const float fq = 1.0f / sqrtf(step_sum(sq, red) + 1e-6f) * (1.0f / sqrtf((float)D)), fk = 1.0f / sqrtf(step_sum(sk, red) + 1e-6f);
        const float beta = sigmoid(p.beta.p[r * p.beta.pitch + h]);
        float read = 0.0f; // (the sums above end behind a barrier: q, k, v, g and gate are there)
#pragma unroll
        for (int i = 0; i < R; i++) {
            const uint32_t d = min(group + i * groups, D);
            S[i] *= g[d];
            read = fmaf(S[i], k[d] * fk, read);
        }
        part[tid] = read;
        __syncthreads();
        read = 0.0f;
        for (uint32_t i = 0; i < groups; i++) read += part[i * lanes + c];
        const float u = c < V ? beta * (v[c] - read) : 0.0f;
        float y = 0.0f;
#pragma unroll
        for (int i = 0; i < R; i++) {
            const uint32_t d = min(group + i * groups, D);
            S[i] = fmaf(k[d] * fk, u, S[i]);
            y = fmaf(S[i], q[d] * fq, y);
        }
        __syncthreads();
        part[tid] = y;
        __syncthreads();
        y = 0.0f;
        if (group == 0)
            for (uint32_t i = 0; i < groups; i++) y += part[i * lanes + c];
        const float f = 1.0f / sqrtf(step_sum(group == 0 && c < V ? y * y : 0.0f, red) / (float)V + p.eps);
        if (group == 0 && c < V) p.out[r * p.heads * V + h * V + c] = y * f * p.norm[c] * gate[c];
        __syncthreads(); // the next token overwrites what this one reads
    }
    keep_inputs(p, b, h);
#pragma unroll
    for (int i = 0; i < R; i++) {
        const uint32_t d = group + i * groups;
        if (d < D && c < V) p.state_out[sb + (int64_t)d * V + c] = S[i];
    }
}

// gate: [B * S, heads * vdim]; in place on `o`
__global__ __launch_bounds__(kThreads) void delta_finish_kernel(const DeltaPlan p, const float *__restrict__ gate, float *__restrict__ o, const uint64_t heads_in_all) {
    const uint64_t w = (uint64_t)blockIdx.x * kWaves + (threadIdx.x >> 6);
    if (w >= heads_in_all) return;
    const uint32_t lane = threadIdx.x & 63;
    float *x = o + w * p.vdim;
    const float *gt = gate + w * p.vdim;
    float ss = 0.0f;
    for (uint32_t d = lane; d < p.vdim; d += 64) ss = fmaf(x[d], x[d], ss);
    const float f = 1.0f / sqrtf(wave_sum(ss) / (float)p.vdim + p.eps);
    for (uint32_t d = lane; d < p.vdim; d += 64) x[d] = x[d] * f * p.norm[d] * sigmoid(gt[d]);
}

int launched(const char *what) {
    const hipError_t e = hipGetLastError();
    return e == hipSuccess ? CG_OK : hip_fail(e, what);
}

struct Scratch {
    cg_backend *be;
    std::vector<std::pair<void *, size_t>> mem;
    explicit Scratch(cg_backend *b) : be(b) {}
    int get(size_t floats, float **p) {
        void *m;
        size_t cls;
        int rc = be->pool.alloc(floats * 4, &m, &cls);
        if (!rc) mem.emplace_back(m, cls);
        *p = static_cast<float *>(m);
        return rc;
    }
    ~Scratch() {
        for (auto &a : mem) be->pool.free(a.first, a.second);
    }
};

// x[rows, rank] . w^T [n, rank] in f32
int low_rank(cg_backend *be, const Rows &x, uint32_t rows, const float *w, uint32_t n, uint32_t rank, float *y) {
    if (few_rows_slots(rows, (uint64_t)staged_pitch(rank) * 4)) {
        ProductInput in;
        in.x = x;
        in.k1 = in.k = rank;
        Weight wt;
        wt.p = w;
        wt.pitch = rank;
        wt.n = n;
        wt.k = rank;
        return launch_few_rows_linear(be, in, rows, wt, nullptr, 1.0f, y);
    }
    Buffer bx, bw, bo; // borrowed memory
    cg_tensor tx, tw, to;
    auto view = [&](cg_tensor &t, Buffer &b, const void *p, int64_t d0, int64_t d1, int64_t s0, int64_t s1) {
        b.be = be;
        b.ptr = const_cast<void *>(p);
        t.be = be;
        t.buf = &b;
        t.rank = 2;
        t.dims[0] = d0;
        t.dims[1] = d1;
        t.strides[0] = s0;
        t.strides[1] = s1;
    };
    view(tx, bx, x.p, rows, rank, x.pitch, 1);
    view(tw, bw, w, rank, n, 1, rank);
    view(to, bo, y, rows, n, n, 1);
    const int rc = launch_matmul(be, &tx, &tw, &to);
    tx.buf = tw.buf = to.buf = nullptr;
    return rc;
}

} // namespace

namespace {

// Whether a step's state fits the registers of one workgroup per head, and how many threads stand side by side on a row.
bool step_shape(const DeltaPlan &p, uint32_t *lanes, uint32_t *rows) {
    if (p.S > kFewRows || p.vdim > (uint32_t)kStepThreads) return false;
    *lanes = 1;
    while (*lanes < p.vdim) *lanes *= 2;
    const uint32_t groups = kStepThreads / *lanes;
    *rows = (p.dim + groups - 1) / groups;
    return *rows <= 64;
}

template <int TPW, int CT> int scan(cg_backend *be, const DeltaPlan &p, const ChunkArrays &a, const float *state) {
    const size_t lds = (size_t)(2 * chunk_lds_floats(64 * TPW) + CT * 4 * 2 * 64 * 4) * 4;
    if (lds > (64 << 10)) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(&delta_scan_kernel<TPW, CT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return hip_fail(e, "hipFuncSetAttribute");
    }
    hipLaunchKernelGGL((delta_scan_kernel<TPW, CT>), dim3((p.vdim + 16 * CT - 1) / (16 * CT), p.heads, p.B), dim3(CT * 256), lds, be->stream, p, a, state, p.out);
    return CG_OK;
}
template <int CT> int scan(cg_backend *be, const DeltaPlan &p, const ChunkArrays &a, const float *state) {
    switch (a.dp / 64) {
    case 1: return scan<1, CT>(be, p, a, state);
    case 2: return scan<2, CT>(be, p, a, state);
    case 3: return scan<3, CT>(be, p, a, state);
    default: return scan<4, CT>(be, p, a, state);
    }
}

} // namespace

int launch_channel_delta(cg_backend *be, const DeltaPlan &p) {
    const uint32_t rows = p.B * p.S, vc = p.heads * p.vdim, hd = p.heads * p.dim;
    const double flop = (double)p.heads * p.dim * p.vdim * 7.0; // a token's decay, read, write and read-out
    uint32_t lanes = 0, held = 0;
    if (step_shape(p, &lanes, &held)) {
        ProfScope prof(be, CG_K_RECURRENCE, flop * rows);
        const dim3 grid(p.heads, p.B);
#define CG_STEP(R)                                                                                                          \
    if (p.taps == 4) hipLaunchKernelGGL((delta_step_kernel<R, 4>), grid, dim3(kStepThreads), 0, be->stream, p, lanes);      \
    else hipLaunchKernelGGL((delta_step_kernel<R, 0>), grid, dim3(kStepThreads), 0, be->stream, p, lanes)
        if (held <= 4) { CG_STEP(4); }
        else if (held <= 16) { CG_STEP(16); }
        else if (held <= 32) { CG_STEP(32); }
        else { CG_STEP(64); }
#undef CG_STEP
        return launched("channel_delta step");
    }
    Scratch mem(be);
    float *decay, *gate;
    if (int rc = mem.get((size_t)rows * hd, &decay)) return rc;
    if (int rc = mem.get((size_t)rows * vc, &gate)) return rc;
    if (int rc = low_rank(be, p.decay, rows, p.decay_w, hd, p.decay_rank, decay)) return rc;
    if (int rc = low_rank(be, p.gate, rows, p.gate_w, vc, p.gate_rank, gate)) return rc;
    ChunkArrays a{};
    a.dp = (p.dim + 63) / 64 * 64;
    // tokens in parts whose chunks' matrices stay within about 512 MB
    const uint32_t chunks = (p.S + kChunk - 1) / kChunk;
    const size_t per_chunk = (size_t)p.B * p.heads * (chunk_floats(a.dp) + kChunk * p.vdim);
    const uint32_t most = (uint32_t)std::max<size_t>(1, std::min<size_t>(chunks, (128u << 20) / per_chunk));
    if (int rc = mem.get((size_t)p.B * p.heads * most * chunk_floats(a.dp), &a.mats)) return rc;
    if (int rc = mem.get((size_t)p.B * p.heads * most * kChunk * p.vdim, &a.u)) return rc;
    const bool wide = (uint64_t)p.B * p.heads * ((p.vdim + 31) / 32) >= (uint64_t)be->compute_units && p.vdim > 16;
    for (uint32_t c0 = 0; c0 < chunks; c0 += most) {
        a.first = c0 * kChunk;
        a.chunks = std::min(most, chunks - c0);
        const uint32_t tokens = std::min(a.chunks * kChunk, p.S - a.first);
        ProfScope prof(be, CG_K_RECURRENCE, flop * tokens * p.B);
        const size_t lds = (size_t)3 * kChunk * (a.dp + 4) * 4;
        const dim3 grid(a.chunks, p.heads, p.B);
        if (p.taps == 4) hipLaunchKernelGGL((delta_chunk_kernel<4>), grid, dim3(kThreads), lds, be->stream, p, a, decay);
        else hipLaunchKernelGGL((delta_chunk_kernel<0>), grid, dim3(kThreads), lds, be->stream, p, a, decay);
        const float *state = c0 ? p.state_out : p.state;
        if (int rc = wide ? scan<2>(be, p, a, state) : scan<1>(be, p, a, state)) return rc;
    }
    const uint64_t n = (uint64_t)rows * p.heads;
    hipLaunchKernelGGL(delta_finish_kernel, dim3((uint32_t)((n + kWaves - 1) / kWaves)), dim3(kThreads), 0, be->stream, p, gate, p.out, n);
    return launched("channel_delta");
}

} // namespace cg
