// Helpers of the recurrent mixers' kernels: fp32 MFMA fragments, LDS-only barrier, scans.
#pragma once

#include "elem.h"

namespace mlop {

// lane l: A[row l & 15][k = l >> 4], B[k = l >> 4][col l & 15]; C / D row 4 (l >> 4) + i, col l & 15.  Four
// of them with the k index taken as 4 (l >> 4) + i make a 16-deep product whose A operand is a 4-vector
// per lane and whose B operand has the accumulator's own layout.
__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mfma_f32x16(const f32x4& a, const f32x4& b, f32x4 c) {
#pragma unroll
  for (int i = 0; i < 4; ++i) c = mfma_f32(a[i], b[i], c);
  return c;
}

// workgroup barrier for LDS hand-offs: global loads and stores stay in flight across it
__device__ __forceinline__ void lds_sync() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  raw_barrier();
}

__device__ __forceinline__ float exp2_f(float x) { return __builtin_amdgcn_exp2f(x); }
constexpr float kLog2E = 1.4426950408889634f;

__device__ __forceinline__ float softplus_f(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ float sigmoid_acc(float x) { return 1.f / (1.f + expf(-x)); }

// four elements p[0 .. 3], those past `left` zero; `vec`: the address is aligned to four elements
template <typename E>
__device__ __forceinline__ f32x4 ld4m(const E* p, int left, bool vec) {
  float v[4] = {0.f, 0.f, 0.f, 0.f};
  if (vec && left >= 4) {
    ldn<4>(p, v);
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (e < left) v[e] = ld1(p + e);
  }
  return f32x4{v[0], v[1], v[2], v[3]};
}

}  // namespace mlop
