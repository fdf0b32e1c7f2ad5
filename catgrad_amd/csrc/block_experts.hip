// Mixtures of experts (cg_block_residual): which experts a token uses, and the products with their weights.
//
//   a few rows    expert_first_kernel   a workgroup per (row, choice, columns): the choice made anew by every workgroup, then
//                                       its columns of both first matrices streamed and the activation
//                 expert_second_kernel  a wave per output columns: the mixer's output product and the chosen experts' second
//                                       matrices, the residual sum in the store
//   many rows     route_kernel          a wave per token: the choice, and a place for the token in each chosen expert's list
//                 route_lists_kernel    the lists, and which tile of which expert every workgroup of the products takes
//                 expert_tile_kernel    products on the matrix instructions: rows gathered through the lists, the activation
//                                       in the store of the first; 16 / 32 values of k per row and stage by loads straight
//                                       into a ring of LDS stages, one barrier a stage
#include "block_stream.hpp"

#include <algorithm>

namespace cg {
namespace {

constexpr int kThreads = 256, kWaves = 4;

__device__ __forceinline__ uint32_t round_bf16(float v) { return asu(v) + 0x7FFFu + ((asu(v) >> 16) & 1u); } // (bits above 15 hold the pattern)
__device__ __forceinline__ float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float activation(float g, float u, float limit, float slope) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g * (u + 1.0f) / (1.0f + __builtin_amdgcn_exp2f(-1.44269504088896341f * slope * g));
}

// ---- the choice ------------------------------------------------------------------------------------------------------
// Every score is ranked against those it competes with: first a group's members, then the groups, then the members of the
// groups that count.  LDS: route_floats(experts, groups) floats.  Thread t of N; `chosen` and `weight` (LDS) are there after
// the last barrier, which is the whole workgroup's.
__host__ __device__ constexpr uint32_t route_floats(uint32_t experts, uint32_t groups) { return 2 * experts + 3 * groups; }
__device__ __forceinline__ bool beats(float a, uint32_t i, float b, uint32_t j) { return a > b || (a == b && i < j); }

template <int N>
__device__ void choose_experts(const ExpertsPlan &p, uint32_t row, float *lds, uint32_t *chosen, float *weight, const uint32_t t) {
    float *choice = lds, *own = lds + p.experts, *worth = own + p.experts; // worth: [groups][2], then [groups] whether it counts
    float *counts = worth + 2 * p.groups;
    const uint32_t size = p.experts / p.groups;
    for (uint32_t e = t; e < p.experts; e += N) {
        const float s = sigmoid(p.logits[(int64_t)row * p.experts + e]);
        own[e] = s;
        choice[e] = p.correction ? s + p.correction[e] : s;
    }
    for (uint32_t g = t; g < p.groups; g += N) worth[2 * g] = worth[2 * g + 1] = 0.0f; // (a group of one member)
    for (uint32_t i = t; i < p.top; i += N) { // (scores that are not numbers leave places untaken)
        chosen[i] = 0;
        weight[i] = 0.0f;
    }
    __syncthreads();
    if (p.keep < p.groups) {
        for (uint32_t e = t; e < p.experts; e += N) {
            const uint32_t g = e / size, first = g * size;
            const float mine = choice[e];
            uint32_t rank = 0;
            for (uint32_t j = first; j < first + size; j++) rank += beats(choice[j], j, mine, e);
            if (rank < 2) worth[2 * g + rank] = mine;
        }
        __syncthreads();
        for (uint32_t g = t; g < p.groups; g += N) {
            const float mine = worth[2 * g] + worth[2 * g + 1];
            uint32_t rank = 0;
            for (uint32_t j = 0; j < p.groups; j++) rank += beats(worth[2 * j] + worth[2 * j + 1], j, mine, g);
            counts[g] = rank < p.keep ? 1.0f : 0.0f;
        }
        __syncthreads();
        for (uint32_t e = t; e < p.experts; e += N)
            if (counts[e / size] == 0.0f) choice[e] = -INFINITY;
        __syncthreads();
    }
    for (uint32_t e = t; e < p.experts; e += N) {
        const float mine = choice[e];
        uint32_t rank = 0;
#pragma unroll 4
        for (uint32_t j = 0; j < p.experts; j++) rank += beats(choice[j], j, mine, e);
        if (rank < p.top) {
            chosen[rank] = e;
            weight[rank] = own[e];
        }
    }
    __syncthreads();
}

// ---- a few rows ------------------------------------------------------------------------------------------------------
// blockIdx.x: columns (four waves, one after the other), blockIdx.y: row * top + choice
template <bool BF16, bool VEC, int STEPS>
__global__ __launch_bounds__(kThreads) void expert_first_kernel(const ExpertsPlan p, const uint32_t per_wave, float *__restrict__ hidden, uint32_t *__restrict__ chosen_out) {
    extern __shared__ float lds[];
    typedef Streamed<BF16, VEC> St;
    constexpr uint32_t W = St::W, SPAN = 64 * W;
    const uint32_t row = blockIdx.y / p.top, slot = blockIdx.y - row * p.top, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    uint32_t *chosen = reinterpret_cast<uint32_t *>(lds + route_floats(p.experts, p.groups));
    float *weight = reinterpret_cast<float *>(chosen + p.top);
    // the row of h, this lane's values of it in registers where they fit
    float x[STEPS][W];
    auto take = [&](uint32_t k, float(&o)[W]) { // (clamped; zeros behind the last column)
        const int64_t at = (int64_t)row * p.width + min(k, p.width - W);
        if (p.h_fmt == kFmtBF16) {
#pragma unroll
            for (uint32_t i = 0; i < W; i++) o[i] = asf((uint32_t) static_cast<const uint16_t *>(p.h)[at + i] << 16);
        } else {
            St::input(static_cast<const float *>(p.h), at, o);
        }
#pragma unroll
        for (uint32_t i = 0; i < W; i++) o[i] = k < p.width ? o[i] : 0.0f;
    };
#pragma unroll
    for (int s = 0; s < STEPS; s++) take(s * SPAN + lane * W, x[s]);
    choose_experts<kThreads>(p, row, lds, chosen, weight, threadIdx.x);
    const uint32_t e = chosen[slot];
    const float weigh = weight[slot];
    if (blockIdx.x == 0 && threadIdx.x == 0) chosen_out[blockIdx.y] = e;
    const uint32_t f0 = (blockIdx.x * kWaves + wave) * per_wave;
    constexpr uint32_t EB = BF16 ? 2 : 4;
    for (uint32_t f = f0; f < min(f0 + per_wave, p.ff); f++) {
        const char *g = static_cast<const char *>(p.gate_up) + ((uint64_t)e * 2 * p.ff + f) * p.width * EB, *u = g + (uint64_t)p.ff * p.width * EB;
        float a = 0.0f, b = 0.0f;
        if (p.width <= STEPS * SPAN) {
            St wg[STEPS], wu[STEPS];
#pragma unroll
            for (int s = 0; s < STEPS; s++) { // (clamped: behind the last column x is zero)
                const uint32_t k = min(s * SPAN + lane * W, p.width - W);
                wg[s].load(g, k);
                wu[s].load(u, k);
            }
#pragma unroll
            for (int s = 0; s < STEPS; s++) {
                a = wg[s].dot(x[s], a);
                b = wu[s].dot(x[s], b);
            }
        } else {
            for (uint32_t k = lane * W; k < p.width; k += SPAN) {
                St wg, wu;
                wg.load(g, k);
                wu.load(u, k);
                float v[W];
                take(k, v);
                a = wg.dot(v, a);
                b = wu.dot(v, b);
            }
        }
        a = wave_total(a);
        b = wave_total(b);
        if (lane == 0) hidden[(uint64_t)blockIdx.y * p.ff + f] = weigh * activation(a, b, p.limit, p.slope);
    }
}

// A wave per NC output columns of a row: out = x + scale * (y . w^T + sum over the choices).  The choices' rows and w's are
// walked as one run of pieces (64 lanes' worth), AHEAD of them in flight.
template <bool BF16, bool VEC, int NC>
__global__ __launch_bounds__(kThreads) void expert_second_kernel(const ExpertsPlan p, const float *__restrict__ hidden, const uint32_t *__restrict__ chosen, const Rows x,
                                                                 const Rows y, const Weight w, const float scale, float *__restrict__ out) {
    typedef Streamed<BF16, VEC> St;
    constexpr uint32_t W = St::W, SPAN = 64 * W, EB = BF16 ? 2 : 4;
    constexpr int AHEAD = 4;
    const uint32_t lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), row = blockIdx.y;
    const uint32_t n0 = (blockIdx.x * kWaves + wave) * NC;
    if (n0 >= p.width) return;
    const uint32_t steps = (p.ff + SPAN - 1) / SPAN, wsteps = w.p ? (w.k + SPAN - 1) / SPAN : 0, total = p.top * steps + wsteps;
    float xs[NC], a[NC];
#pragma unroll
    for (int c = 0; c < NC; c++) {
        xs[c] = x.p[(int64_t)row * x.pitch + min(n0 + c, p.width - 1)];
        a[c] = 0.0f;
    }
    const float *yr = y.p + (int64_t)row * y.pitch, *hr = hidden + (uint64_t)row * p.top * p.ff;
    for (uint32_t i0 = 0; i0 < total; i0 += AHEAD) {
        St s[AHEAD][NC];
        float v[AHEAD][W];
#pragma unroll
        for (int e = 0; e < AHEAD; e++) { // (pieces behind the last, and lanes behind a row's end: clamped, and times zero)
            const uint32_t i = min(i0 + e, total - 1), slot = i / steps;
            const bool first = i < p.top * steps;
            const uint32_t k0 = (first ? i - slot * steps : i - p.top * steps) * SPAN + lane * W, K = first ? p.ff : w.k, k = min(k0, K - W);
            const char *d = first ? static_cast<const char *>(p.down) + (uint64_t)chosen[(uint64_t)row * p.top + slot] * p.width * p.ff * EB : static_cast<const char *>(w.p);
            const uint64_t pitch = first ? p.ff : (uint64_t)w.pitch;
#pragma unroll
            for (int c = 0; c < NC; c++) s[e][c].load(d + min(n0 + c, p.width - 1) * pitch * EB, k);
            St::input(first ? hr + slot * p.ff : yr, k, v[e]);
            const bool there = i0 + e < total && k0 < K;
#pragma unroll
            for (uint32_t j = 0; j < W; j++) v[e][j] = there ? v[e][j] : 0.0f;
        }
#pragma unroll
        for (int e = 0; e < AHEAD; e++)
#pragma unroll
            for (int c = 0; c < NC; c++) a[c] = s[e][c].dot(v[e], a[c]);
    }
#pragma unroll
    for (int c = 0; c < NC; c++) {
        const float sum = wave_total(a[c]);
        if (lane == 0 && n0 + c < p.width) out[(uint64_t)row * p.width + n0 + c] = fmaf(scale, sum, xs[c]);
    }
}

// the same for one (row, choice) at a time, of any number: y[row * top + slot, n]
template <bool BF16, bool VEC>
__global__ __launch_bounds__(kThreads) void expert_second_slots_kernel(const ExpertsPlan p, const float *__restrict__ hidden, const uint32_t *__restrict__ chosen,
                                                                       float *__restrict__ y) {
    typedef Streamed<BF16, VEC> St;
    constexpr uint32_t W = St::W, SPAN = 64 * W, EB = BF16 ? 2 : 4;
    const uint32_t lane = threadIdx.x & 63, n = blockIdx.x * kWaves + (threadIdx.x >> 6);
    const uint64_t at = blockIdx.y;
    if (n >= p.width) return;
    const char *d = static_cast<const char *>(p.down) + ((uint64_t)chosen[at] * p.width + n) * p.ff * EB;
    float a = 0.0f;
    for (uint32_t k = lane * W; k < p.ff; k += SPAN) {
        St s;
        s.load(d, k);
        float v[W];
        St::input(hidden + at * p.ff, k, v);
        a = s.dot(v, a);
    }
    a = wave_total(a);
    if (lane == 0) y[at * p.width + n] = a;
}

// ---- many rows -------------------------------------------------------------------------------------------------------
// choice[r * top + slot]: expert, place in its list; count[e]: rows of expert e
struct Routed {
    uint32_t expert, place;
};
// A workgroup takes `run` tokens, a wave one at a time, and its places in the experts' lists in one go.
__host__ __device__ constexpr uint32_t route_wave_floats(const ExpertsPlan &p) { return route_floats(p.experts, p.groups) + 2 * p.top; }
__global__ __launch_bounds__(kThreads) void route_kernel(const ExpertsPlan p, const uint32_t run, Routed *__restrict__ routed, float *__restrict__ weights, uint32_t *__restrict__ count) {
    extern __shared__ float lds[];
    const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r0 = blockIdx.x * run, n = min(run, p.rows - r0);
    float *mine = lds + wave * route_wave_floats(p);
    uint32_t *chosen = reinterpret_cast<uint32_t *>(mine + route_floats(p.experts, p.groups));
    float *weight = reinterpret_cast<float *>(chosen + p.top);
    uint32_t *seen = reinterpret_cast<uint32_t *>(lds + kWaves * route_wave_floats(p)), *base = seen + p.experts, *place = base + p.experts, *whose = place + run * p.top; // [run][top]
    for (uint32_t e = threadIdx.x; e < p.experts; e += kThreads) seen[e] = 0;
    __syncthreads();
    for (uint32_t i = wave; i < run; i += kWaves) { // (the same trips for every wave: the choice has barriers)
        const uint32_t row = r0 + min(i, n - 1);
        choose_experts<64>(p, row, mine, chosen, weight, lane);
        if (i < n)
            for (uint32_t t = lane; t < p.top; t += 64) {
                const uint64_t at = (uint64_t)row * p.top + t;
                weights[at] = weight[t];
                whose[i * p.top + t] = chosen[t];
                place[i * p.top + t] = atomicAdd(seen + chosen[t], 1u);
            }
        __syncthreads();
    }
    for (uint32_t e = threadIdx.x; e < p.experts; e += kThreads) base[e] = seen[e] ? atomicAdd(count + e, seen[e]) : 0;
    __syncthreads();
    for (uint32_t i = threadIdx.x; i < n * p.top; i += kThreads) {
        routed[(uint64_t)r0 * p.top + i] = {whose[i], base[whose[i]] + place[i]};
    }
}
__global__ __launch_bounds__(kThreads) void clear_kernel(uint32_t *p, uint32_t n) {
    const uint32_t i = blockIdx.x * kThreads + threadIdx.x;
    if (i < n) p[i] = 0;
}

// list: the choices (row * top + slot) expert by expert; tiles: {expert, first place in the list, places, -} per tile of TM
// places, and {0, 0, 0} where there is none.  Every workgroup adds the counts up for itself.
__global__ __launch_bounds__(kThreads) void route_lists_kernel(const uint32_t experts, const uint32_t n, const uint32_t tm, const uint32_t max_tiles, const Routed *__restrict__ routed,
                                                               const uint32_t *__restrict__ count, uint32_t *__restrict__ list, uint4 *__restrict__ tiles) {
    extern __shared__ uint32_t start[]; // [experts + 1] places, [experts + 1] tiles
    uint32_t *tile0 = start + experts + 1;
    for (uint32_t e = threadIdx.x; e < experts; e += kThreads) {
        uint32_t a = 0, t = 0;
        for (uint32_t j = 0; j < e; j++) {
            const uint32_t c = count[j];
            a += c;
            t += (c + tm - 1) / tm;
        }
        start[e] = a;
        tile0[e] = t;
    }
    __syncthreads();
    const uint32_t i = blockIdx.x * kThreads + threadIdx.x;
    if (i < n) {
        const Routed r = routed[i];
        list[start[r.expert] + r.place] = i;
    }
    if (blockIdx.x == 0) {
        for (uint32_t e = threadIdx.x; e < experts; e += kThreads) {
            const uint32_t c = count[e];
            for (uint32_t t = 0; t * tm < c; t++) tiles[tile0[e] + t] = make_uint4(e, start[e] + t * tm, min(tm, c - t * tm), 0);
        }
        const uint32_t used = tile0[experts - 1] + (count[experts - 1] + tm - 1) / tm;
        for (uint32_t t = used + threadIdx.x; t < max_tiles; t += kThreads) tiles[t] = make_uint4(0, 0, 0, 0);
    }
}

constexpr uint32_t kTileN = 128, kStages = 4;
typedef float float16v __attribute__((ext_vector_type(16)));
typedef float float4v __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
__device__ const uint32_t kZeros[4] __attribute__((aligned(16))) = {0, 0, 0, 0};

struct ExpertTileArgs {
    const char *x, *w;        // x: rows of the left operand
    const uint32_t *list;
    const uint4 *tiles;
    const float *weights;     // FIRST: per choice
    void *out;                // FIRST: hidden [place in the list, ff], else [choice, N]; in the form of x
    uint32_t N, K;            // FIRST: N = ff
    uint32_t top, tiles_n;
    float limit, slope;
};

// 64 MT x 128 tiles of an expert's rows, four waves of 32 MT x 64 each.  A stage is 64 bytes of k per row, by loads straight
// into LDS in a ring of four: one multiplied, three in flight, one barrier a stage.  A row's four 16-byte columns lie at column
// c ^ ((row >> 2) & 3), so that the lanes that a 128-bit read serves together cover all banks.  FIRST: the tile's 128 weight
// rows are 64 of each first matrix, 32 in turn, so that a lane finds both factors of its activations; the left operand's rows
// come through the list.  f32: lane group g supplies k = 4 (2 c + g) + t to the t-th of four instructions.
template <bool BF16, bool FIRST, int MT> __global__ __launch_bounds__(kThreads) void expert_tile_kernel(const ExpertTileArgs a) {
    constexpr uint32_t TM = 64 * MT, A_BYTES = TM * 64, STAGE = A_BYTES + kTileN * 64, EB = BF16 ? 2 : 4, STAGE_K = 64 / EB;
    constexpr uint32_t OUT_N = FIRST ? 64 : 128; // output columns of a tile
    extern __shared__ float lds_dyn[];
    typedef __attribute__((address_space(3))) char lds_char;
    lds_char *const lds = (lds_char *)lds_dyn;
    // (tiles in order: the empty ones at the end cost every XCD the same, and an XCD's tiles share two columns of weights)
    const uint32_t tile = blockIdx.x / a.tiles_n, n0 = (blockIdx.x - tile * a.tiles_n) * OUT_N;
    const uint4 job = a.tiles[tile];
    const uint32_t m = job.z, nk = (a.K + STAGE_K - 1) / STAGE_K;
    if (m == 0) return;
    const uint32_t wave = __builtin_amdgcn_readfirstlane(threadIdx.x / 64), lane = threadIdx.x % 64;
    const uint32_t wm = (wave / 2) * 32 * MT, wn = (wave % 2) * 64, li = lane % 32, lg = lane / 32;
    const uint64_t pitch = (uint64_t)a.K * EB;
    const char *const w = a.w + (uint64_t)job.x * (FIRST ? 2 : 1) * a.N * pitch;

    const char *src[MT + 2];
    const uint32_t col = (lane % 4) ^ ((lane >> 4) & 3); // the logical 16-byte column this lane fetches; (row >> 2) & 3 with row = 16 n + lane / 4
#pragma unroll
    for (int q = 0; q < MT; q++) {
        const uint32_t place = job.y + min((wave * MT + q) * 16 + lane / 4, m - 1);
        src[q] = a.x + (uint64_t)(FIRST ? a.list[place] / a.top : place) * pitch + col * 16;
    }
#pragma unroll
    for (int q = 0; q < 2; q++) {
        const uint32_t r = (wave * 2 + q) * 16 + lane / 4;
        const uint32_t n = FIRST ? min(n0 + (r >> 6) * 32 + (r & 31), a.N - 1) + ((r >> 5) & 1) * a.N : min(n0 + r, a.N - 1);
        src[MT + q] = w + n * pitch + col * 16;
    }
    auto issue = [&](const uint32_t stage, const uint32_t at) {
        const uint32_t k0 = stage * STAGE_K;
        const bool outside = k0 + col * (16 / EB) >= a.K;
#pragma unroll
        for (int q = 0; q < MT + 2; q++) {
            const char *p = src[q] + (uint64_t)k0 * EB;
            if (outside) p = reinterpret_cast<const char *>(kZeros);
            lds_char *const l = lds + at * STAGE + (q < MT ? (wave * MT + q) * 1024 : A_BYTES + (wave * 2 + q - MT) * 1024);
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void *)p, (__attribute__((address_space(3))) void *)l, 16, 0, 0);
        }
    };
    const uint32_t sw = (li >> 2) & 3;
    auto frag = [&](const uint32_t base, const uint32_t c) {
        return *reinterpret_cast<const __attribute__((address_space(3))) float4v *>(lds + base + li * 64 + ((c ^ sw) * 16));
    };
    float16v acc[MT][2];
#pragma unroll
    for (int i = 0; i < MT; i++)
#pragma unroll
        for (int j = 0; j < 2; j++)
#pragma unroll
            for (int v = 0; v < 16; v++) acc[i][j][v] = 0.0f;

    for (uint32_t s = 0; s < kStages - 1; s++) issue(min(s, nk - 1), s);
    for (uint32_t kt = 0; kt < nk; kt++) {
        constexpr uint32_t n = 2 * (MT + 2); // two younger stages may be in flight
        asm volatile("" ::: "memory");
        __builtin_amdgcn_s_waitcnt(0x0070 | n); // vmcnt(n) lgkmcnt(0)
        __builtin_amdgcn_s_barrier();
        asm volatile("" ::: "memory");
        issue(min(kt + kStages - 1, nk - 1), (kt + kStages - 1) % kStages);
        const uint32_t base = (kt % kStages) * STAGE;
#pragma unroll
        for (int c = 0; c < 2; c++) {
            float4v fa[MT], fb[2];
#pragma unroll
            for (int i = 0; i < MT; i++) fa[i] = frag(base + (wm + i * 32) * 64, c * 2 + lg);
#pragma unroll
            for (int j = 0; j < 2; j++) fb[j] = frag(base + A_BYTES + (wn + j * 32) * 64, c * 2 + lg);
#pragma unroll
            for (int i = 0; i < MT; i++)
#pragma unroll
                for (int j = 0; j < 2; j++) {
                    if constexpr (BF16) {
                        acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, fa[i]), __builtin_bit_cast(bf16x8, fb[j]), acc[i][j], 0, 0, 0);
                    } else {
#pragma unroll
                        for (int t = 0; t < 4; t++) acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x2f32(fa[i][t], fb[j][t], acc[i][j], 0, 0, 0);
                    }
                }
        }
    }
    asm volatile("" ::: "memory");
    __builtin_amdgcn_s_waitcnt(0x0070); // no load may write LDS that another workgroup gets

    // the instruction's result: row 8 (v / 4) + 4 lg + v % 4, column li
#pragma unroll
    for (int i = 0; i < MT; i++)
#pragma unroll
        for (int v = 0; v < 16; v++) {
            const uint32_t r = wm + i * 32 + 8 * (v / 4) + 4 * lg + (v % 4);
            if (r >= m) continue;
            const uint32_t place = job.y + r, choice = a.list[place];
            if constexpr (FIRST) {
                const uint32_t f = n0 + (wave % 2) * 32 + li;
                if (f >= a.N) continue;
                const float h = a.weights[choice] * activation(acc[i][0][v], acc[i][1][v], a.limit, a.slope);
                if constexpr (BF16) static_cast<uint16_t *>(a.out)[(uint64_t)place * a.N + f] = (uint16_t)(round_bf16(h) >> 16);
                else static_cast<float *>(a.out)[(uint64_t)place * a.N + f] = h;
            } else {
#pragma unroll
                for (int j = 0; j < 2; j++) {
                    const uint32_t n = n0 + wn + j * 32 + li;
                    if (n >= a.N) continue;
                    if constexpr (BF16) static_cast<uint16_t *>(a.out)[(uint64_t)choice * a.N + n] = (uint16_t)(round_bf16(acc[i][j][v]) >> 16);
                    else static_cast<float *>(a.out)[(uint64_t)choice * a.N + n] = acc[i][j][v];
                }
            }
        }
}

int launched(const char *what) {
    const hipError_t e = hipGetLastError();
    return e == hipSuccess ? CG_OK : hip_fail(e, what);
}
bool aligned16(const void *p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

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

size_t route_bytes(const ExpertsPlan &p) { return (route_floats(p.experts, p.groups) + 2 * (size_t)p.top) * 4; }
constexpr uint32_t kMaxRun = 16;
size_t many_route_bytes(const ExpertsPlan &p) { return (kWaves * (size_t)route_wave_floats(p) + 2 * (size_t)p.experts + 2 * (size_t)kMaxRun * p.top) * 4; }
bool vector_rows(const ExpertsPlan &p) {
    const uint32_t vw = p.fmt == kFmtBF16 ? 8 : 4;
    return p.width % vw == 0 && p.ff % vw == 0 && aligned16(p.gate_up) && aligned16(p.down) && aligned16(p.h);
}
double first_bytes(const ExpertsPlan &p, double used) { return used * 2.0 * p.ff * p.width * (p.fmt == kFmtBF16 ? 2.0 : 4.0); }

template <bool BF16, bool FIRST, int MT> int launch_tiles(cg_backend *be, const ExpertTileArgs &a, uint32_t tiles) {
    const size_t lds = (size_t)kStages * (64 * MT + kTileN) * 64;
    hipLaunchKernelGGL((expert_tile_kernel<BF16, FIRST, MT>), dim3(tiles * a.tiles_n), dim3(kThreads), lds, be->stream, a);
    return launched("expert_tiles");
}

} // namespace

int launch_experts_first(cg_backend *be, const ExpertsPlan &p, float *hidden, uint32_t *chosen) {
    const uint32_t pairs = p.rows * p.top;
    if (route_bytes(p) > (64u << 10)) return fail(CG_ERR_UNSUPPORTED, "experts: more than the kernels hold");
    const bool bf16 = p.fmt == kFmtBF16, vec = vector_rows(p);
    ProfScope prof(be, CG_K_GEMM_SKINNY, first_bytes(p, pairs));
    // columns of a wave: enough workgroups for the device, not many more
    const uint32_t per = std::max(1u, (uint32_t)((uint64_t)pairs * p.ff / ((uint64_t)be->compute_units * 8 * kWaves)));
    const uint32_t per_wave = std::min(per, 8u);
    const size_t lds = route_bytes(p);
    hipStream_t s = be->stream;
    for (uint32_t first = 0; first < p.rows;) { // (the grid's y extent)
        const uint32_t n = std::min(p.rows - first, std::max(1u, 65535 / p.top));
        ExpertsPlan q = p;
        q.rows = n;
        q.h = static_cast<const char *>(p.h) + (uint64_t)first * p.width * (p.h_fmt == kFmtBF16 ? 2 : 4);
        q.logits = p.logits + (uint64_t)first * p.experts;
        float *hid = hidden + (uint64_t)first * p.top * p.ff;
        uint32_t *ch = chosen + (uint64_t)first * p.top;
        const dim3 grid((p.ff + kWaves * per_wave - 1) / (kWaves * per_wave), n * p.top);
        const uint32_t steps = (p.width + 64 * (bf16 ? 8 : 4) - 1) / (64 * (bf16 ? 8 : 4));
#define CG_FIRST(BF, VE, ST) hipLaunchKernelGGL((expert_first_kernel<BF, VE, ST>), grid, dim3(kThreads), lds, s, q, per_wave, hid, ch)
#define CG_FIRST_ST(BF)                        \
    if (!vec) CG_FIRST(BF, false, 1);          \
    else if (steps <= 1) CG_FIRST(BF, true, 1); \
    else if (steps <= 2) CG_FIRST(BF, true, 2); \
    else if (steps <= 4) CG_FIRST(BF, true, 4); \
    else CG_FIRST(BF, true, 8)
        if (bf16) { CG_FIRST_ST(true); }
        else { CG_FIRST_ST(false); }
#undef CG_FIRST_ST
#undef CG_FIRST
        first += n;
    }
    return launched("expert_first");
}

int launch_experts_second(cg_backend *be, const ExpertsPlan &p, const float *hidden, const uint32_t *chosen, const Rows &x, const Rows &y, const Weight *w, float scale,
                          float *out) {
    const bool bf16 = p.fmt == kFmtBF16;
    bool vec = vector_rows(p);
    Weight none;
    if (w) {
        if (w->fmt != p.fmt) return fail(CG_ERR_DTYPE, "experts: the output product's weights have another dtype");
        const uint32_t vw = bf16 ? 8 : 4;
        vec = vec && w->k % vw == 0 && w->pitch % vw == 0 && aligned16(w->p) && y.pitch % 4 == 0 && aligned16(y.p);
    }
    ProfScope prof(be, CG_K_GEMM_SKINNY, first_bytes(p, p.rows * p.top) / 2 + (w ? (double)w->n * w->k * (bf16 ? 2.0 : 4.0) : 0.0));
    const bool two = vec && (uint64_t)p.rows * p.width >= 16ull * be->compute_units; // columns of a wave
    const uint32_t per = kWaves * (two ? 2 : 1);
    const dim3 grid((p.width + per - 1) / per, p.rows);
#define CG_SECOND(BF, VE)                                                                                                                                            \
    {                                                                                                                                                                \
        if (two) hipLaunchKernelGGL((expert_second_kernel<BF, VE, VE ? 2 : 1>), grid, dim3(kThreads), 0, be->stream, p, hidden, chosen, x, y, w ? *w : none, scale, out); \
        else hipLaunchKernelGGL((expert_second_kernel<BF, VE, 1>), grid, dim3(kThreads), 0, be->stream, p, hidden, chosen, x, y, w ? *w : none, scale, out);           \
    }
    if (bf16 && vec) CG_SECOND(true, true)
    else if (bf16) CG_SECOND(true, false)
    else if (vec) CG_SECOND(false, true)
    else CG_SECOND(false, false)
#undef CG_SECOND
    return launched("expert_second");
}

int launch_experts(cg_backend *be, const ExpertsPlan &p, float *y, int *y_fmt) {
    *y_fmt = kFmtWords;
    const bool bf16 = p.fmt == kFmtBF16, vec = vector_rows(p);
    const uint64_t n = (uint64_t)p.rows * p.top;
    if (n > 0x7FFFFFFFull || p.experts > 4096) return fail(CG_ERR_UNSUPPORTED, "experts: more than the kernels hold");
    const bool tiled = vec && many_route_bytes(p) <= (64u << 10) && (p.h_fmt == kFmtBF16) == bf16 && aligned16(p.h);
    if (!tiled) { // shapes that do not lie in 16-byte pieces: every choice on its own
        Scratch hid(be), ch(be);
        if (int rc = hid.get(n * p.ff * 4)) return rc;
        if (int rc = ch.get(n * 4)) return rc;
        float *hidden = static_cast<float *>(hid.p);
        uint32_t *chosen = static_cast<uint32_t *>(ch.p);
        if (int rc = launch_experts_first(be, p, hidden, chosen)) return rc;
        ProfScope prof(be, CG_K_GEMM_SKINNY, first_bytes(p, n) / 2);
        for (uint64_t at = 0; at < n; at += 65535) {
            const dim3 grid((p.width + kWaves - 1) / kWaves, (uint32_t)std::min<uint64_t>(n - at, 65535));
#define CG_SLOTS(BF, VE) hipLaunchKernelGGL((expert_second_slots_kernel<BF, VE>), grid, dim3(kThreads), 0, be->stream, p, hidden + at * p.ff, chosen + at, y + at * p.width)
            if (bf16 && vec) CG_SLOTS(true, true);
            else if (bf16) CG_SLOTS(true, false);
            else if (vec) CG_SLOTS(false, true);
            else CG_SLOTS(false, false);
#undef CG_SLOTS
        }
        return launched("expert_slots");
    }
    *y_fmt = bf16 ? kFmtBF16 : kFmtWords;
    // lists
    const bool low = n <= 64ull * p.experts; // few rows per expert: short tiles
    const uint32_t tm = low ? 64 : 128, max_tiles = (uint32_t)(n / tm + std::min<uint64_t>(p.experts, n));
    Scratch mem(be), hid(be);
    const size_t bytes = n * sizeof(Routed) + n * 4 + n * 4 + (size_t)p.experts * 4 + 16 + (size_t)max_tiles * 16;
    if (int rc = mem.get(bytes)) return rc;
    if (int rc = hid.get(n * p.ff * (bf16 ? 2 : 4))) return rc;
    uint4 *tiles = static_cast<uint4 *>(mem.p);
    Routed *routed = reinterpret_cast<Routed *>(tiles + max_tiles);
    float *weights = reinterpret_cast<float *>(routed + n);
    uint32_t *list = reinterpret_cast<uint32_t *>(weights + n), *count = list + n;
    {
        ProfScope prof(be, CG_K_GATHER, 4.0 * p.rows * p.experts + 20.0 * n);
        hipLaunchKernelGGL(clear_kernel, dim3((p.experts + kThreads - 1) / kThreads), dim3(kThreads), 0, be->stream, count, p.experts);
        const uint32_t run = std::min(kMaxRun, (uint32_t)kWaves * std::max(1u, p.rows / (4 * be->compute_units * kWaves)));
        hipLaunchKernelGGL(route_kernel, dim3((p.rows + run - 1) / run), dim3(kThreads), many_route_bytes(p), be->stream, p, run, routed, weights, count);
        hipLaunchKernelGGL(route_lists_kernel, dim3((uint32_t)((n + kThreads - 1) / kThreads)), dim3(kThreads), (size_t)(p.experts + 1) * 8, be->stream, p.experts, (uint32_t)n, tm,
                           max_tiles, routed, count, list, tiles);
        if (int rc = launched("route")) return rc;
    }
    ExpertTileArgs a{};
    a.x = static_cast<const char *>(p.h);
    a.w = static_cast<const char *>(p.gate_up);
    a.list = list;
    a.tiles = tiles;
    a.weights = weights;
    a.out = hid.p;
    a.N = p.ff;
    a.K = p.width;
    a.top = p.top;
    a.tiles_n = (p.ff + 63) / 64;
    a.limit = p.limit;
    a.slope = p.slope;
    int rc;
    {
        ProfScope prof(be, CG_K_GEMM_MFMA, 4.0 * (double)n * p.ff * p.width);
        rc = bf16 ? (low ? launch_tiles<true, true, 1>(be, a, max_tiles) : launch_tiles<true, true, 2>(be, a, max_tiles))
                  : (low ? launch_tiles<false, true, 1>(be, a, max_tiles) : launch_tiles<false, true, 2>(be, a, max_tiles));
    }
    if (rc) return rc;
    a.x = static_cast<const char *>(hid.p);
    a.w = static_cast<const char *>(p.down);
    a.out = y;
    a.N = p.width;
    a.K = p.ff;
    a.tiles_n = (p.width + kTileN - 1) / kTileN;
    ProfScope prof(be, CG_K_GEMM_MFMA, 2.0 * (double)n * p.ff * p.width);
    return bf16 ? (low ? launch_tiles<true, false, 1>(be, a, max_tiles) : launch_tiles<true, false, 2>(be, a, max_tiles))
                : (low ? launch_tiles<false, false, 1>(be, a, max_tiles) : launch_tiles<false, false, 2>(be, a, max_tiles));
}

} // namespace cg
