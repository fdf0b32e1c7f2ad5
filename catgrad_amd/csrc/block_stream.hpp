// Weight rows streamed through registers by the decoder blocks' kernels for a few rows.
#pragma once

#include "blocks.hpp"
#include "device_utils.hpp"

namespace cg {

__device__ __forceinline__ float bf16_lo(uint32_t w) { return asf(w << 16); }
__device__ __forceinline__ float bf16_hi(uint32_t w) { return asf(w & 0xFFFF0000u); }

// A lane's piece of a row of words or bfloat16 patterns: 16 bytes (VEC) or one value, and its product with activations.
template <bool BF16, bool VEC> struct Streamed {
    static constexpr uint32_t W = VEC ? (BF16 ? 8 : 4) : 1;
    uint4 v;
    __device__ __forceinline__ void load(const void *row, uint32_t k) {
        if constexpr (VEC) {
            typedef uint32_t u4 __attribute__((ext_vector_type(4)));
            const u4 t = __builtin_nontemporal_load(reinterpret_cast<const u4 *>(static_cast<const char *>(row) + (uint64_t)k * (BF16 ? 2 : 4)));
            v = make_uint4(t[0], t[1], t[2], t[3]);
        } else {
            v.x = BF16 ? (uint32_t)static_cast<const uint16_t *>(row)[k] << 16 : static_cast<const uint32_t *>(row)[k];
        }
    }
    __device__ __forceinline__ float dot(const float (&x)[W], float s) const {
        if constexpr (!VEC) {
            return fmaf(asf(v.x), x[0], s);
        } else if constexpr (BF16) {
            const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
            for (int i = 0; i < 4; i++) {
                s = fmaf(bf16_lo(w[i]), x[2 * i], s);
                s = fmaf(bf16_hi(w[i]), x[2 * i + 1], s);
            }
            return s;
        } else {
            s = fmaf(asf(v.x), x[0], s);
            s = fmaf(asf(v.y), x[1], s);
            s = fmaf(asf(v.z), x[2], s);
            return fmaf(asf(v.w), x[3], s);
        }
    }
    static __device__ __forceinline__ void input(const float *x, uint64_t k, float (&o)[W]) {
        if constexpr (VEC) {
#pragma unroll
            for (uint32_t i = 0; i < W; i += 4) {
                const float4 t = *reinterpret_cast<const float4 *>(x + k + i);
                o[i] = t.x, o[i + 1] = t.y, o[i + 2] = t.z, o[i + 3] = t.w;
            }
        } else {
            o[0] = x[k];
        }
    }
};

} // namespace cg
