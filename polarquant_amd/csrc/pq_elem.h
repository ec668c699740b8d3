// Elements of a tensor in any of the three dtypes (F16, BF16, F32) as floats, and a wavefront's sum.
#pragma once
#include "pq_device.h"

namespace pq {

struct F32 {};

template <typename T> struct Elem { using type = uint16_t; };
template <> struct Elem<F32> { using type = float; };
template <typename T> using elem_t = typename Elem<T>::type;

template <typename T> __device__ __forceinline__ float ld1(const elem_t<T>* p) {
    if constexpr (__is_same(T, F32)) return *p; else return lo2f<T>(*p);
}
template <typename T> __device__ __forceinline__ elem_t<T> cv1(float f) {
    if constexpr (__is_same(T, F32)) return f; else return f2lo<T>(f);
}
// V consecutive elements (V 1 or 4; for 4 the address is a multiple of 4 elements)
template <typename T, int V> __device__ __forceinline__ void ldv(const void* base, size_t i, float (&o)[V]) {
    const elem_t<T>* p = static_cast<const elem_t<T>*>(base) + i;
    if constexpr (V == 1) {
        o[0] = ld1<T>(p);
    } else if constexpr (__is_same(T, F32)) {
        const float4 v = *reinterpret_cast<const float4*>(p);
        o[0] = v.x; o[1] = v.y; o[2] = v.z; o[3] = v.w;
    } else {
        const uint2 v = *reinterpret_cast<const uint2*>(p);
        o[0] = lo2f<T>(static_cast<uint16_t>(v.x & 0xffffu)); o[1] = lo2f<T>(static_cast<uint16_t>(v.x >> 16));
        o[2] = lo2f<T>(static_cast<uint16_t>(v.y & 0xffffu)); o[3] = lo2f<T>(static_cast<uint16_t>(v.y >> 16));
    }
}
template <typename T, int V> __device__ __forceinline__ void stv(void* base, size_t i, const float (&o)[V]) {
    elem_t<T>* p = static_cast<elem_t<T>*>(base) + i;
    if constexpr (V == 1) {
        *p = cv1<T>(o[0]);
    } else if constexpr (__is_same(T, F32)) {
        *reinterpret_cast<float4*>(p) = make_float4(o[0], o[1], o[2], o[3]);
    } else {
        *reinterpret_cast<uint2*>(p) = make_uint2(static_cast<uint32_t>(f2lo<T>(o[0])) | (static_cast<uint32_t>(f2lo<T>(o[1])) << 16),
                                                  static_cast<uint32_t>(f2lo<T>(o[2])) | (static_cast<uint32_t>(f2lo<T>(o[3])) << 16));
    }
}

// sum over the wavefront, in every lane: rotations inside rows of 16 lanes, then the four rows' sums through scalars
__device__ __forceinline__ float wave_sum(float v) {
    v += __uint_as_float(row_rotate<8>(__float_as_uint(v)));
    v += __uint_as_float(row_rotate<4>(__float_as_uint(v)));
    v += __uint_as_float(row_rotate<2>(__float_as_uint(v)));
    v += __uint_as_float(row_rotate<1>(__float_as_uint(v)));
    return (readlane_f(v, 0) + readlane_f(v, 16)) + (readlane_f(v, 32) + readlane_f(v, 48));
}

}  // namespace pq
