// Short causal convolution per channel with silu, over a ragged step:
//
//   out[t, c] = silu(b[c] + sum_j w[c, j] x[t - (taps - 1) + j, c]),   zeros before a sequence's start
//
// A sequence's last taps - 1 inputs are its state (`tail`, fp32, oldest first).  A thread owns VEC
// channels of up to kTile tokens and slides the window through registers.  The workgroup of a portion's
// first tile reads the old tail and then writes the new one, so that nothing else touches it.
#include "elem.h"
#include "mixers.h"

namespace mlop {

namespace {

constexpr int kTile = 16;

__device__ __forceinline__ float silu_c(float x) { return x / (1.f + __expf(-x)); }

}  // namespace

// ROWS: one-token rows (blockIdx.x: row); else (item, tile of kTile tokens in blockIdx.z)
template <typename E, int VEC, int TAPS, bool ROWS>
__global__ void __launch_bounds__(256) short_conv_kernel(ConvArgs a, StepRows r) {
  constexpr int P = TAPS - 1, PM = P ? P : 1;
  const int s = ROWS ? r.rows[blockIdx.x] : r.item_seq[blockIdx.x];
  const int t0 = ROWS ? 0 : r.item_t0[blockIdx.x] + (int)blockIdx.z * kTile;
  const int ql = r.q_len[s], ctx = r.ctx_len[s], q0 = r.q_start[s];
  const int c = ((int)blockIdx.y * 256 + (int)threadIdx.x) * VEC;
  const int n = ROWS ? 1 : min(kTile, min(ql, r.item_t0[blockIdx.x] + r.chunk) - t0);
  if (c >= a.C || n <= 0) return;
  E* out = reinterpret_cast<E*>(a.out) + (size_t)(q0 + t0) * a.C + c;
  if (ctx < ql || s >= r.n_slots) {  // graph padding
    float z[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) z[e] = 0.f;
    for (int t = 0; t < n; ++t) stn<VEC>(out + (size_t)t * a.C, z);
    return;
  }
  const E* x = reinterpret_cast<const E*>(a.x) + (size_t)q0 * a.ldx + c;
  float* tail = a.tail + ((size_t)s * P) * a.C + c;
  float w[TAPS][VEC], bias[VEC], win[PM][VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) {
    bias[e] = a.b ? a.b[c + e] : 0.f;
#pragma unroll
    for (int j = 0; j < TAPS; ++j) w[j][e] = a.w[(size_t)(c + e) * TAPS + j];
  }
#pragma unroll
  for (int j = 0; j < P; ++j) {
    const int t = t0 - P + j;  // token of the portion; before it: the tail
    if (t >= 0) {
      ldn<VEC>(x + (size_t)t * a.ldx, win[j]);
    } else if (ctx == ql) {
#pragma unroll
      for (int e = 0; e < VEC; ++e) win[j][e] = 0.f;
    } else {
      ldn<VEC>(tail + (size_t)(P + t) * a.C, win[j]);
    }
  }
  if (t0 == 0 && P > 0) {  // the new tail: last P of [old tail | portion]
    float nt[PM][VEC];
#pragma unroll
    for (int j = 0; j < P; ++j) {
      const int t = ql - P + j;
      if (t >= 0) {
        ldn<VEC>(x + (size_t)t * a.ldx, nt[j]);
      } else if (ctx == ql) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) nt[j][e] = 0.f;
      } else {
        ldn<VEC>(tail + (size_t)(P + t) * a.C, nt[j]);
      }
    }
#pragma unroll
    for (int j = 0; j < P; ++j) stn<VEC>(tail + (size_t)j * a.C, nt[j]);
  }
  constexpr int NB = ROWS ? 1 : kTile;
  float in[NB][VEC];
#pragma unroll
  for (int t = 0; t < NB; ++t) ldn<VEC>(x + (size_t)(t0 + min(t, n - 1)) * a.ldx, in[t]);
#pragma unroll
  for (int t = 0; t < NB; ++t) {
    float o[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      o[e] = bias[e];
#pragma unroll
      for (int j = 0; j < TAPS; ++j) {
        const int k = t - P + j;  // compile-time after unrolling
        o[e] = fmaf(w[j][e], k >= 0 ? in[k < 0 ? 0 : k][e] : win[k < 0 ? P + k : 0][e], o[e]);
      }
      o[e] = silu_c(o[e]);
    }
    if (t < n) stn<VEC>(out + (size_t)t * a.C, o);
  }
}

template <typename E, int VEC, int TAPS>
static void conv_taps(const ConvArgs& a, const StepRows& r, hipStream_t st) {
  const int cb = cdiv(cdiv(a.C, VEC), 256);
  if (r.n_rows) short_conv_kernel<E, VEC, TAPS, true><<<dim3(r.n_rows, cb), 256, 0, st>>>(a, r);
  if (r.n_items) short_conv_kernel<E, VEC, TAPS, false><<<dim3(r.n_items, cb, cdiv(r.chunk, kTile)), 256, 0, st>>>(a, r);
}

template <typename E, int VEC>
static void conv_vec(const ConvArgs& a, const StepRows& r, hipStream_t st) {
  switch (a.taps) {
#define MLOP_TAPS(N) case N: conv_taps<E, VEC, N>(a, r, st); break;
    MLOP_TAPS(1) MLOP_TAPS(2) MLOP_TAPS(3) MLOP_TAPS(4)
#undef MLOP_TAPS
    default: break;
  }
}

template <typename E>
static void conv_any(const ConvArgs& a, const StepRows& r, hipStream_t st) {
  switch (a.taps) {  // long kernels: one channel per thread
#define MLOP_TAPS(N) case N: conv_taps<E, 1, N>(a, r, st); break;
    MLOP_TAPS(1) MLOP_TAPS(2) MLOP_TAPS(3) MLOP_TAPS(4) MLOP_TAPS(5) MLOP_TAPS(6) MLOP_TAPS(7) MLOP_TAPS(8)
    MLOP_TAPS(9) MLOP_TAPS(10) MLOP_TAPS(11) MLOP_TAPS(12) MLOP_TAPS(13) MLOP_TAPS(14) MLOP_TAPS(15) MLOP_TAPS(16)
#undef MLOP_TAPS
    default: break;
  }
}

void launch_short_conv(const ConvArgs& a, const StepRows& s, bool f32, hipStream_t st) {
  const bool al = ((reinterpret_cast<uintptr_t>(a.x) | reinterpret_cast<uintptr_t>(a.out) |
                    reinterpret_cast<uintptr_t>(a.tail)) & 15) == 0;
  const bool v4 = al && a.C % 4 == 0 && a.ldx % 4 == 0 && a.taps <= 4;
  if (f32) {
    if (v4) conv_vec<float, 4>(a, s, st); else conv_any<float>(a, s, st);
  } else {
    if (v4) conv_vec<uint16_t, 4>(a, s, st); else conv_any<uint16_t>(a, s, st);
  }
}

}  // namespace mlop
