// Products of bfloat16 patterns with the sums in 32-bit, for prompts that do not fill the device with 256 x 256 tiles:
// y[M, N] = x[M, K] . w[N, K]^T, cut along k as well when there are few tiles.
#include "blocks.hpp"
#include "device_utils.hpp"

#include <algorithm>

namespace cg {
namespace {

constexpr int kThreads = 256;
constexpr uint32_t kTileN = 128, kStages = 4, kStageK = 32, kXcds = 8, kGroupM = 8;
typedef float float16v __attribute__((ext_vector_type(16)));
typedef float float4v __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

struct TileArgs {
    const char *x, *w;
    float *y;                  // split s of y at y + s * M * N
    uint32_t M, N, K;
    uint32_t x_pitch, w_pitch; // bytes
    uint32_t k_part;           // values of k per split, a multiple of kStageK
};

__device__ const uint32_t kZeros[4] __attribute__((aligned(16))) = {0, 0, 0, 0};

// 64 MT x 128 tiles, four waves of 32 MT x 64 each.  A stage is 64 bytes of k per row, fetched by loads straight into LDS in
// a ring of four: one multiplied, three in flight, one barrier a stage.  A row's four 16-byte columns lie at column
// c ^ ((row >> 2) & 3), so that the lanes that a 128-bit read serves together cover all banks; a load instruction of a wave
// fills 16 rows in lane order.  Rows beyond the edge are clamped, columns beyond K come from a block of zeros.
template <int MT> __global__ __launch_bounds__(kThreads) void bf16_tile_kernel(const TileArgs a) {
    constexpr uint32_t TM = 64 * MT, A_BYTES = TM * 64, STAGE = A_BYTES + kTileN * 64;
    extern __shared__ float lds_dyn[];
    typedef __attribute__((address_space(3))) char lds_char;
    lds_char *const lds = (lds_char *)lds_dyn;

    // a run of tiles per XCD, down a column of kGroupM row tiles first
    const uint32_t tiles_n = (a.N + kTileN - 1) / kTileN, tiles_m = (a.M + TM - 1) / TM, ntiles = tiles_m * tiles_n;
    const uint32_t xcd = blockIdx.x % kXcds, q8 = ntiles / kXcds, r8 = ntiles % kXcds;
    const uint32_t lin = xcd * q8 + min(xcd, r8) + blockIdx.x / kXcds;
    const uint32_t group = lin / (kGroupM * tiles_n), in_group = lin % (kGroupM * tiles_n), first_m = group * kGroupM;
    const uint32_t gsize = min(tiles_m - first_m, kGroupM);
    const uint32_t m0 = (first_m + in_group % gsize) * TM, n0 = (in_group / gsize) * kTileN;
    const uint32_t k_first = blockIdx.y * a.k_part, k_end = min(k_first + a.k_part, a.K), nk = (k_end - k_first + kStageK - 1) / kStageK;

    const uint32_t wave = __builtin_amdgcn_readfirstlane(threadIdx.x / 64), lane = threadIdx.x % 64;
    const uint32_t wm = (wave / 2) * 32 * MT, wn = (wave % 2) * 64, li = lane % 32, lg = lane / 32;

    // this lane's part of the wave's loads of a stage: MT of x, two of w; `col`: the logical 16-byte column it fetches
    uint32_t off[MT + 2];
    const uint32_t col = (lane % 4) ^ ((lane >> 4) & 3); // ((row >> 2) & 3 with row = 16 n + lane / 4)
#pragma unroll
    for (int q = 0; q < MT; q++) off[q] = min(m0 + (wave * MT + q) * 16 + lane / 4, a.M - 1) * a.x_pitch + col * 16;
#pragma unroll
    for (int q = 0; q < 2; q++) off[MT + q] = min(n0 + (wave * 2 + q) * 16 + lane / 4, a.N - 1) * a.w_pitch + col * 16;
    auto issue = [&](const uint32_t stage, const uint32_t place) {
        const uint32_t k0 = k_first + stage * kStageK;
        const bool tail = k0 + kStageK > a.K, outside = k0 + col * 8 >= a.K;
#pragma unroll
        for (int q = 0; q < MT + 2; q++) {
            const char *p = (q < MT ? a.x : a.w) + (uint64_t)k0 * 2 + off[q];
            if (tail && outside) p = reinterpret_cast<const char *>(kZeros);
            lds_char *const l = lds + place * STAGE + (q < MT ? (wave * MT + q) * 1024 : A_BYTES + (wave * 2 + q - MT) * 1024);
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void *)p, (__attribute__((address_space(3))) void *)l, 16, 0, 0);
        }
    };
    const uint32_t sw = (li >> 2) & 3;
    auto frag = [&](const uint32_t base, const uint32_t c) {
        return __builtin_bit_cast(bf16x8, *reinterpret_cast<const __attribute__((address_space(3))) float4v *>(lds + base + li * 64 + ((c ^ sw) * 16)));
    };

    float16v acc[MT][2];
#pragma unroll
    for (int i = 0; i < MT; i++)
#pragma unroll
        for (int j = 0; j < 2; j++)
#pragma unroll
            for (int v = 0; v < 16; v++) acc[i][j][v] = 0.0f;

    // (behind the last stage the last one is asked for again: one count of loads in flight, and a place that nobody reads)
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
            bf16x8 fa[MT], fb[2];
#pragma unroll
            for (int i = 0; i < MT; i++) fa[i] = frag(base + (wm + i * 32) * 64, c * 2 + lg);
#pragma unroll
            for (int j = 0; j < 2; j++) fb[j] = frag(base + A_BYTES + (wn + j * 32) * 64, c * 2 + lg);
#pragma unroll
            for (int i = 0; i < MT; i++)
#pragma unroll
                for (int j = 0; j < 2; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fa[i], fb[j], acc[i][j], 0, 0, 0);
        }
    }
    asm volatile("" ::: "memory");
    __builtin_amdgcn_s_waitcnt(0x0070); // no load may write LDS that another workgroup gets

    float *const y = a.y + (uint64_t)blockIdx.y * a.M * a.N;
#pragma unroll
    for (int i = 0; i < MT; i++)
#pragma unroll
        for (int j = 0; j < 2; j++) {
            const uint32_t n = n0 + wn + j * 32 + li;
            if (n >= a.N) continue;
#pragma unroll
            for (int v = 0; v < 16; v++) { // the instruction's result: row 8 (v / 4) + 4 lg + v % 4, column li
                const uint32_t m = m0 + wm + i * 32 + 8 * (v / 4) + 4 * lg + (v % 4);
                if (m < a.M) y[(uint64_t)m * a.N + n] = acc[i][j][v];
            }
        }
}

// y[e] = the parts' sum, in their order
__global__ __launch_bounds__(kThreads) void sum_parts_kernel(const float4v *part, float4v *y, uint32_t parts, uint64_t n4) {
    const uint64_t i = (uint64_t)blockIdx.x * kThreads + threadIdx.x;
    if (i >= n4) return;
    float4v v = __builtin_nontemporal_load(part + i);
    for (uint32_t s = 1; s < parts; s++) v += __builtin_nontemporal_load(part + s * n4 + i);
    y[i] = v;
}

int launched(const char *what) {
    const hipError_t e = hipGetLastError();
    return e == hipSuccess ? CG_OK : hip_fail(e, what);
}

} // namespace

int launch_bf16_tiles(cg_backend *be, const void *x, uint32_t rows, const Weight &w, float *y) {
    const uint64_t x_bytes = (uint64_t)rows * w.k * 2, w_bytes = (uint64_t)w.n * (uint64_t)w.pitch * 2;
    if (!takes_bf16_tiles(rows, w) || reinterpret_cast<uintptr_t>(x) % 16) return kDeclined;
    const bool low = rows <= 64;
    const uint32_t tm = low ? 64 : 128;
    const uint64_t tiles = (uint64_t)((rows + tm - 1) / tm) * ((w.n + kTileN - 1) / kTileN);
    if (x_bytes >= (1ull << 32) || w_bytes >= (1ull << 32) || tiles > 0x7FFFFFFFull) return kDeclined;
    TileArgs a{};
    a.x = static_cast<const char *>(x);
    a.w = static_cast<const char *>(w.p);
    a.M = rows;
    a.N = w.n;
    a.K = w.k;
    a.x_pitch = w.k * 2;
    a.w_pitch = (uint32_t)(w.pitch * 2);
    // two workgroups per compute unit, each with at least 256 values of k; the same shape always gets the same cut
    const uint64_t mn = (uint64_t)rows * w.n, room = 2 * (uint64_t)be->compute_units;
    uint32_t splits = mn % 4 ? 1 : (uint32_t)std::max<uint64_t>(1, std::min<uint64_t>({room / tiles, w.k / 256, 16}));
    a.k_part = ((w.k + splits - 1) / splits + kStageK - 1) / kStageK * kStageK;
    splits = (w.k + a.k_part - 1) / a.k_part;
    ProfScope prof(be, CG_K_GEMM_MFMA, 2.0 * (double)mn * w.k);
    void *parts = nullptr;
    size_t cls = 0;
    if (splits > 1)
        if (int rc = be->pool.alloc(mn * splits * 4, &parts, &cls)) return rc;
    a.y = splits > 1 ? static_cast<float *>(parts) : y;
    const dim3 grid((uint32_t)tiles, splits);
    const size_t lds = (size_t)kStages * (tm + kTileN) * 64;
    if (low) hipLaunchKernelGGL((bf16_tile_kernel<1>), grid, dim3(kThreads), lds, be->stream, a);
    else hipLaunchKernelGGL((bf16_tile_kernel<2>), grid, dim3(kThreads), lds, be->stream, a);
    if (splits > 1) {
        hipLaunchKernelGGL(sum_parts_kernel, dim3((uint32_t)((mn / 4 + kThreads - 1) / kThreads)), dim3(kThreads), 0, be->stream,
                           static_cast<const float4v *>(parts), reinterpret_cast<float4v *>(y), splits, mn / 4);
        be->pool.free(parts, cls); // stream-ordered
    }
    return launched("bf16_tiles");
}

bool takes_bf16_tiles(uint32_t rows, const Weight &w) {
    return rows > 0 && w.fmt == kFmtBF16 && w.k % 8 == 0 && w.pitch % 8 == 0 && reinterpret_cast<uintptr_t>(w.p) % 16 == 0;
}

} // namespace cg
