// Sums over the sixteen lanes of a row of a wave by moves inside the vector unit, the same bits in each of them; the sum of a
// product's parts; softplus.
#pragma once
#include "common.h"

namespace arle {

template <int CTRL>
__device__ __forceinline__ float row_move(float v) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
__device__ __forceinline__ float row_sum16(float v) {
  v += row_move<0xB1>(v);    // quad_perm [1, 0, 3, 2]
  v += row_move<0x4E>(v);    // quad_perm [2, 3, 0, 1]
  v += row_move<0x141>(v);   // row_half_mirror
  v += row_move<0x140>(v);   // row_mirror
  return v;
}

// The sum of `parts` numbers `stride` apart in ascending order, eight loads in flight, none under a condition.
__device__ __forceinline__ float sum_parts(const float* p, int parts, long long stride) {
  float s = 0.f;
  for (int i0 = 0; i0 < parts; i0 += 8) {
    float e[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) e[u] = p[min(i0 + u, parts - 1) * stride];
#pragma unroll
    for (int u = 0; u < 8; ++u) s += i0 + u < parts ? e[u] : 0.f;
  }
  return s;
}

__device__ __forceinline__ float softplus_f(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

}  // namespace arle
