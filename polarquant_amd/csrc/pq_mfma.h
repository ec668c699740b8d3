// Matrix-core products and the packing of their 16-bit operands, shared by the attention kernels.
#pragma once
#include "pq_elem.h"

namespace pq {

typedef float floatx4_a __attribute__((ext_vector_type(4)));
typedef float floatx16_a __attribute__((ext_vector_type(16)));
typedef uint32_t u32x4_a __attribute__((ext_vector_type(4)));
typedef uint32_t u32x2_a __attribute__((ext_vector_type(2)));
typedef _Float16 half8_a __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x8_a __attribute__((ext_vector_type(8)));
typedef short short4_a __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) short4_a lds_short4;
typedef __attribute__((address_space(3))) u32x4_a lds_u32x4;

template <typename T> __device__ __forceinline__ floatx4_a mma16(u32x4_a a, u32x4_a b, floatx4_a c);
template <> __device__ __forceinline__ floatx4_a mma16<F16>(u32x4_a a, u32x4_a b, floatx4_a c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(half8_a, a), __builtin_bit_cast(half8_a, b), c, 0, 0, 0);
}
template <> __device__ __forceinline__ floatx4_a mma16<BF16>(u32x4_a a, u32x4_a b, floatx4_a c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_a, a), __builtin_bit_cast(bf16x8_a, b), c, 0, 0, 0);
}
template <typename T> __device__ __forceinline__ floatx16_a mma32(u32x4_a a, u32x4_a b, floatx16_a c);
template <> __device__ __forceinline__ floatx16_a mma32<F16>(u32x4_a a, u32x4_a b, floatx16_a c) {
    return __builtin_amdgcn_mfma_f32_32x32x16_f16(__builtin_bit_cast(half8_a, a), __builtin_bit_cast(half8_a, b), c, 0, 0, 0);
}
template <> __device__ __forceinline__ floatx16_a mma32<BF16>(u32x4_a a, u32x4_a b, floatx16_a c) {
    return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_a, a), __builtin_bit_cast(bf16x8_a, b), c, 0, 0, 0);
}

constexpr float kLog2e = 1.4426950408889634f;
constexpr float kNone = -1.0e30f;         // running maximum before any key
__device__ __forceinline__ float exp2_hw(float x) { return __builtin_amdgcn_exp2f(x); }

template <typename T> __device__ __forceinline__ uint32_t pack2(float a, float b) {
    return static_cast<uint32_t>(f2lo<T>(a)) | (static_cast<uint32_t>(f2lo<T>(b)) << 16);
}

}  // namespace pq
