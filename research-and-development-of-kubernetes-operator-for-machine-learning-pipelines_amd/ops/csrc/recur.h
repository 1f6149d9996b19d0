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

// bf16 operands in the same 16-deep layout (lane: k = 4 (l >> 4) + i), exact products, fp32 sums
using s16x4 = __attribute__((ext_vector_type(4))) short;
__device__ __forceinline__ f32x4 mfma_bf16x16(const u32x2& a, const u32x2& b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(__builtin_bit_cast(s16x4, a), __builtin_bit_cast(s16x4, b), c, 0, 0, 0);
}
// x = hi + mid + lo in bf16, to fp32 accuracy: with an exact bf16 operand, three bf16 products stand for an
// fp32 one
__device__ __forceinline__ void split3(const f32x4& x, u32x2 (&p)[3]) {
  f32x4 r = x;
#pragma unroll
  for (int t = 0; t < 3; ++t) {
    p[t] = u32x2{pack2(r[0], r[1]), pack2(r[2], r[3])};
    if (t < 2) r -= f32x4{lo_bf(p[t][0]), hi_bf(p[t][0]), lo_bf(p[t][1]), hi_bf(p[t][1])};
  }
}

// A decode step's states at this size pass through the caches without staying there: they would not be
// there at the next step, and written lines left behind are written back under the next kernel.
constexpr size_t kStreamBytes = 100u << 20;
template <bool NT, int N>
__device__ __forceinline__ void ld_state(const float* p, float (&v)[N]) {
  if constexpr (NT) ldn_nt<N>(p, v); else ldn<N>(p, v);
}
template <bool NT, int N>
__device__ __forceinline__ void st_state(float* p, const float (&v)[N]) {
  if constexpr (NT) stn_nt<N>(p, v); else stn<N>(p, v);
}

// workgroup barrier for LDS hand-offs: global loads and stores stay in flight across it
__device__ __forceinline__ void lds_sync() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  raw_barrier();
}

__device__ __forceinline__ float exp2_f(float x) { return __builtin_amdgcn_exp2f(x); }
constexpr float kLog2E = 1.4426950408889634f;

__device__ __forceinline__ float softplus_f(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
// to a few fp32 ulp (of 1 for tanh), by the hardware's exp2 and reciprocal
__device__ __forceinline__ float sigmoid_hw(float x) { return __builtin_amdgcn_rcpf(1.f + exp2_f(-kLog2E * x)); }
__device__ __forceinline__ float tanh_hw(float x) { return 1.f - 2.f * __builtin_amdgcn_rcpf(1.f + exp2_f(2.f * kLog2E * x)); }

// inclusive running sum over each row of 16 lanes
__device__ __forceinline__ float scan16(float x) {
#define MLOP_SHR(N)                                                                                            \
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x110 + N /* row_shr */, 0xF, 0xF, true))
  MLOP_SHR(1);
  MLOP_SHR(2);
  MLOP_SHR(4);
  MLOP_SHR(8);
#undef MLOP_SHR
  return x;
}

// Work units dealt to the 8 XCDs in contiguous ranges (workgroups go round them by their index), so that
// neighbours share an L2.  Grid: xcd_grid(units); -1: no unit.
constexpr int kXcds = 8;
__host__ __device__ inline int xcd_grid(int units) { return (units + kXcds - 1) / kXcds * kXcds; }
__device__ __forceinline__ int xcd_unit(int id, int units) {
  const int per = (units + kXcds - 1) / kXcds, u = (id % kXcds) * per + id / kXcds;
  return u < units ? u : -1;
}

// four elements as stored (see Raw8); the address is aligned to four elements if `vec`
template <typename E>
struct Raw4 {
  E v[4];
  __device__ __forceinline__ void load(const E* p, int last, bool vec) {  // p[min(e, last)]
    if (vec) {
      if constexpr (sizeof(E) == 2) {
        const u32x2 t = *reinterpret_cast<const u32x2*>(p);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = (E)(t[e >> 1] >> (16 * (e & 1)));
      } else {
        const f32x4 t = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = (E)t[e];
      }
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = p[min(e, last)];
    }
  }
  __device__ __forceinline__ f32x4 f(int n) const {  // the first n, zeros behind them
    return f32x4{n > 0 ? ld1(&v[0]) : 0.f, n > 1 ? ld1(&v[1]) : 0.f, n > 2 ? ld1(&v[2]) : 0.f, n > 3 ? ld1(&v[3]) : 0.f};
  }
};

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

// Operands are kept as stored and converted where they are used, not where they are loaded, so that a
// block's loads stay in flight together.  Eight consecutive elements; `last`: p[min(e, last)].
template <typename E>
struct Raw8;
template <>
struct Raw8<uint16_t> {
  u32x4 v;
  template <bool VEC>
  __device__ __forceinline__ void load(const uint16_t* p, int last) {
    if constexpr (VEC) {
      v = *reinterpret_cast<const u32x4*>(p);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = (uint32_t)p[min(2 * e, last)] | (uint32_t)p[min(2 * e + 1, last)] << 16;
    }
  }
  __device__ __forceinline__ f32x4 f(int k) const {  // elements 4 k .. + 3
    return f32x4{lo_bf(v[2 * k]), hi_bf(v[2 * k]), lo_bf(v[2 * k + 1]), hi_bf(v[2 * k + 1])};
  }
};
template <>
struct Raw8<float> {
  f32x4 v[2];
  template <bool VEC>
  __device__ __forceinline__ void load(const float* p, int last) {
    if constexpr (VEC) {
      v[0] = *reinterpret_cast<const f32x4*>(p);
      v[1] = *reinterpret_cast<const f32x4*>(p + 4);
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e >> 2][e & 3] = p[min(e, last)];
    }
  }
  __device__ __forceinline__ f32x4 f(int k) const { return v[k]; }
};

}  // namespace mlop
