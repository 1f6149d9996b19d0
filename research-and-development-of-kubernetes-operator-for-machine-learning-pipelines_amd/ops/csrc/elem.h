// Element access for kernels of two element types (bf16 as uint16_t, and float): single elements
// and aligned vectors, converted to and from fp32.
#pragma once

#include "common.h"

namespace mlop {

__device__ __forceinline__ float ld1(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float ld1(const float* p) { return *p; }
__device__ __forceinline__ void st1(uint16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void st1(float* p, float v) { *p = v; }

// N consecutive elements, N a power of two <= 8; the address is N-element aligned
template <int N>
__device__ __forceinline__ void ldn(const float* p, float (&v)[N]) {
  if constexpr (N % 4 == 0) {
#pragma unroll
    for (int i = 0; i < N; i += 4) {
      const f32x4 t = *reinterpret_cast<const f32x4*>(p + i);
#pragma unroll
      for (int j = 0; j < 4; ++j) v[i + j] = t[j];
    }
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = p[i];
  }
}
template <int N>
__device__ __forceinline__ void ldn(const uint16_t* p, float (&v)[N]) {
  if constexpr (N == 8) {
    const u32x4 t = *reinterpret_cast<const u32x4*>(p);
#pragma unroll
    for (int j = 0; j < 4; ++j) v[2 * j] = lo_bf(t[j]), v[2 * j + 1] = hi_bf(t[j]);
  } else if constexpr (N == 4) {
    const u32x2 t = *reinterpret_cast<const u32x2*>(p);
#pragma unroll
    for (int j = 0; j < 2; ++j) v[2 * j] = lo_bf(t[j]), v[2 * j + 1] = hi_bf(t[j]);
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = bf2f(p[i]);
  }
}
template <int N>
__device__ __forceinline__ void stn(float* p, const float (&v)[N]) {
  if constexpr (N % 4 == 0) {
#pragma unroll
    for (int i = 0; i < N; i += 4)
      *reinterpret_cast<f32x4*>(p + i) = f32x4{v[i], v[i + 1], v[i + 2], v[i + 3]};
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) p[i] = v[i];
  }
}
template <int N>
__device__ __forceinline__ void stn(uint16_t* p, const float (&v)[N]) {
  if constexpr (N == 8) {
    *reinterpret_cast<u32x4*>(p) =
        u32x4{pack2(v[0], v[1]), pack2(v[2], v[3]), pack2(v[4], v[5]), pack2(v[6], v[7])};
  } else if constexpr (N == 4) {
    *reinterpret_cast<u32x2*>(p) = u32x2{pack2(v[0], v[1]), pack2(v[2], v[3])};
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) p[i] = f2bf(v[i]);
  }
}

// four (or one) floats that stream through: read or written once per launch, not kept in the caches
template <int N>
__device__ __forceinline__ void ldn_nt(const float* p, float (&v)[N]) {
  if constexpr (N == 4) {
    const f32x4 t = __builtin_nontemporal_load(reinterpret_cast<const f32x4*>(p));
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = t[j];
  } else {
#pragma unroll
    for (int j = 0; j < N; ++j) v[j] = __builtin_nontemporal_load(p + j);
  }
}
template <int N>
__device__ __forceinline__ void stn_nt(float* p, const float (&v)[N]) {
  if constexpr (N == 4) {
    __builtin_nontemporal_store(f32x4{v[0], v[1], v[2], v[3]}, reinterpret_cast<f32x4*>(p));
  } else {
#pragma unroll
    for (int j = 0; j < N; ++j) __builtin_nontemporal_store(v[j], p + j);
  }
}

}  // namespace mlop
