// Helpers of the recurrences over matrix states (retention, state-space duality): sums over a few neighbouring lanes, the
// 32-bit matrix product, four elements of a row at a time.
#pragma once

#include "common.h"

__device__ __forceinline__ float lane_xor1(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0xB1, 0xf, 0xf, false));
}
__device__ __forceinline__ float lane_xor2(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x4E, 0xf, 0xf, false));
}
__device__ __forceinline__ float lane_half_mirror(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x141, 0xf, 0xf, false));
}
// The sum over eight neighbouring lanes; each of them gets the same bits.
__device__ __forceinline__ float sum_of_eight_lanes(float v) {
  v += lane_xor1(v);
  v += lane_xor2(v);
  v += lane_half_mirror(v);
  return v;
}

template <typename T> struct alignas(4 * sizeof(T)) Four { T e[4]; };

typedef float f32x4_t __attribute__((ext_vector_type(4)));
// One step of depth 4 of a 16 x 16 product in 32-bit.  Operands: lane (n16, g4) = (lane % 16, lane / 16) holds row (of b:
// column) n16 at depth g4; results: rows 4 g4 + i, column n16.
__device__ __forceinline__ f32x4_t mfma_f32(float a, float b, f32x4_t c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
