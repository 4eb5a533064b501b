// Operands of the 16-row matrix instructions, read straight from memory, for both storage types.
#pragma once

#include "common.h"

namespace st {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float floatx4 __attribute__((ext_vector_type(4)));

// Operands in the matrix instructions' layout: lane (r16, g) holds, of row r16, the elements
// k0 + 8g .. 8g+7 (bfloat16, one product of depth 32) or k0 + 4g .. 4g+3 (float, four products
// of depth 4, the u-th taking element u of every lane).
template <typename T> struct Frag;
template <> struct Frag<bf16_t> {
    static constexpr int kDepth = 32, kLane = 8;
    bf16x8 v;
    __device__ inline void load_whole(const bf16_t* p) { v = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(p)); }
    __device__ inline void load(const bf16_t* row, int k, int K, bool ok, bool vec) {
        if (ok && vec && k + 8 <= K) {
            v = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(row + k));
        } else {
            uint16_t e[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) e[i] = (ok && k + i < K) ? row[k + i].bits : (uint16_t)0;
            v = __builtin_bit_cast(bf16x8, make_uint4(e[0] | ((uint32_t)e[1] << 16), e[2] | ((uint32_t)e[3] << 16),
                                                      e[4] | ((uint32_t)e[5] << 16), e[6] | ((uint32_t)e[7] << 16)));
        }
    }
    __device__ static inline floatx4 mma(const Frag& a, const Frag& b, floatx4 c) {
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
    }
};
template <> struct Frag<float> {
    static constexpr int kDepth = 16, kLane = 4;
    float v[4];
    __device__ inline void load_whole(const float* p) {
        const float4 x = *reinterpret_cast<const float4*>(p);
        v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w;
    }
    __device__ inline void load(const float* row, int k, int K, bool ok, bool vec) {
        if (ok && vec && k + 4 <= K) {
            const float4 x = *reinterpret_cast<const float4*>(row + k);
            v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w;
        } else {
#pragma unroll
            for (int i = 0; i < 4; ++i) v[i] = (ok && k + i < K) ? row[k + i] : 0.f;
        }
    }
    __device__ static inline floatx4 mma(const Frag& a, const Frag& b, floatx4 c) {
#pragma unroll
        for (int u = 0; u < 4; ++u) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.v[u], b.v[u], c, 0, 0, 0);
        return c;
    }
};

}  // namespace st
