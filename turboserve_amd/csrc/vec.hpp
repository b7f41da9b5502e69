// Loads and stores of VEC neighbouring elements (one access of 8 or 16 bytes where VEC is 4), in 32-bit on the
// device's side; the address must then be aligned to the access.
#pragma once

#include "common.hpp"

typedef __bf16 vec_bf16x2 __attribute__((ext_vector_type(2)));
typedef float vec_f32x2 __attribute__((ext_vector_type(2)));

template <typename P, int VEC>
__device__ __forceinline__ void load_vec(const P* p, float (&v)[VEC]) {
  if constexpr (VEC == 4 && sizeof(P) == 4) {
    const float4 raw = *reinterpret_cast<const float4*>(p);
    v[0] = raw.x; v[1] = raw.y; v[2] = raw.z; v[3] = raw.w;
  } else if constexpr (VEC == 4) {
    const uint2 raw = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(raw.x << 16);
    v[1] = __uint_as_float(raw.x & 0xffff0000u);
    v[2] = __uint_as_float(raw.y << 16);
    v[3] = __uint_as_float(raw.y & 0xffff0000u);
  } else {
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = to_float(p[e]);
  }
}

template <typename T, int VEC>
__device__ __forceinline__ void store_vec(T* p, const float (&v)[VEC]) {
  if constexpr (VEC == 4 && sizeof(T) == 4) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  } else if constexpr (VEC == 4) {
    // (Round to nearest even, two elements an instruction.)
    const vec_bf16x2 low = __builtin_convertvector(vec_f32x2{v[0], v[1]}, vec_bf16x2);
    const vec_bf16x2 high = __builtin_convertvector(vec_f32x2{v[2], v[3]}, vec_bf16x2);
    *reinterpret_cast<uint2*>(p) = make_uint2(__builtin_bit_cast(uint32_t, low), __builtin_bit_cast(uint32_t, high));
  } else {
#pragma unroll
    for (int e = 0; e < VEC; ++e) p[e] = from_float<T>(v[e]);
  }
}
