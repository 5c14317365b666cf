// Device helpers shared by the recurrent mixers (csrc/kernels/recur.hip, forget.hip).
#pragma once
#include "bfly_common.h"

namespace bfly {

// an input's activation (1: silu); FAST (bf16 inputs): hardware exp and reciprocal
template <bool FAST>
__device__ __forceinline__ float act_in(float v, int act) {
  if (act != 1) return v;
  if (FAST) return v * __builtin_amdgcn_rcpf(1.f + __expf(-v));
  return v / (1.f + expf(-v));
}

// element 4 j .. 4 j + 3 of a row, zeros from n on
template <typename T>
__device__ __forceinline__ f32x4 load4(const T* __restrict__ row, int c, int n, bool vec) {
  typedef T tv __attribute__((ext_vector_type(4)));
  f32x4 r = {0.f, 0.f, 0.f, 0.f};
  if (vec && c + 3 < n) {
    const tv v = *reinterpret_cast<const tv*>(row + c);
#pragma unroll
    for (int e = 0; e < 4; ++e) r[e] = (float)v[e];
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (c + e < n) r[e] = (float)row[c + e];
  }
  return r;
}

__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

template <int CTRL>
__device__ __forceinline__ float dpp_add(float v) {
  return v + __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xF, 0xF, true));
}
// sum over the four lanes of a quad / the sixteen lanes of a row, in every lane
__device__ __forceinline__ float quad_sum(float v) { return dpp_add<0x4E>(dpp_add<0xB1>(v)); }
__device__ __forceinline__ float row16_sum(float v) { return dpp_add<0x140>(dpp_add<0x141>(quad_sum(v))); }

inline bool rows_aligned(const void* p, long ld, size_t esz) {
  return ld % 4 == 0 && reinterpret_cast<uintptr_t>(p) % (4 * esz) == 0;
}

}  // namespace bfly
