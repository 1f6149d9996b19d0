// Hyper-connections: S copies of the residual stream in fp32, read, mixed and written around every
// sublayer, with the RMSNorm of the next sublayer's input in the same pass.
//
//   old streams x_s, sublayer output y:   x_t <- sum_s mix[s, t] x_s + w_out[t] y
//   next sublayer's input:                u = sum_t w_in[t] x_t,   xn = u / rms(u) * norm_w
//
// One workgroup per token.  Each stream element is read once and written once: a thread owns the
// same columns of every stream, so the S x S mix happens in registers, and u waits in LDS for the
// row's root mean square.  The pass is HBM-bound: 8 S W bytes of streams per token plus y and xn.
// The first pass of a step starts every stream from the scaled embedding row instead.
#include "elem.h"
#include "hybrid.h"
#include "launch.h"

namespace mlop {

template <typename E, int NS, int VEC, bool START>
__global__ void __launch_bounds__(1024) hyper_kernel(HyperArgs a) {
  extern __shared__ float u_row[];
  __shared__ float scratch[16];
  constexpr int MAXS = NS ? NS : kMaxStreams;
  const int S = NS ? NS : a.S, W = a.W, row = blockIdx.x;
  float* st = a.streams + (size_t)row * S * W;
  const E* y = reinterpret_cast<const E*>(a.y) + (size_t)row * W;
  if constexpr (START) {
    const long id = min(max(a.ids[row], 0l), a.vocab - 1);
    y = reinterpret_cast<const E*>(a.table) + (size_t)id * W;
  }
  float in_sum = 0.f;
  if constexpr (START) {
    for (int s = 0; s < S; ++s) in_sum += a.w_in[s];
  }
  float ss = 0.f;
  for (int c = threadIdx.x * VEC; c < W; c += blockDim.x * VEC) {
    float yv[VEC], u[VEC];
    ldn<VEC>(y + c, yv);
    if constexpr (START) {
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        yv[e] *= a.embed_scale;
        u[e] = 0.f;
      }
      for (int s = 0; s < S; ++s) {
        const float w = a.w_in[s];
#pragma unroll
        for (int e = 0; e < VEC; ++e) u[e] += w * yv[e];
        stn<VEC>(st + (size_t)s * W + c, yv);
      }
    } else {
      float x[MAXS][VEC];
#pragma unroll
      for (int s = 0; s < (NS ? NS : 1); ++s) ldn<VEC>(st + (size_t)s * W + c, x[s]);
      if constexpr (NS == 0)
        for (int s = 1; s < S; ++s) ldn<VEC>(st + (size_t)s * W + c, x[s]);
#pragma unroll
      for (int e = 0; e < VEC; ++e) u[e] = 0.f;
      auto one = [&](int t) {
        float n[VEC];
        const float wo = a.w_out[t], wi = a.w_in[t];
#pragma unroll
        for (int e = 0; e < VEC; ++e) n[e] = wo * yv[e];
        if constexpr (NS) {
#pragma unroll
          for (int s = 0; s < NS; ++s) {
            const float m = a.mix[s * NS + t];
#pragma unroll
            for (int e = 0; e < VEC; ++e) n[e] = fmaf(m, x[s][e], n[e]);
          }
        } else {
          for (int s = 0; s < S; ++s) {
            const float m = a.mix[s * S + t];
#pragma unroll
            for (int e = 0; e < VEC; ++e) n[e] = fmaf(m, x[s][e], n[e]);
          }
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) u[e] = fmaf(wi, n[e], u[e]);
        if (a.store) stn<VEC>(st + (size_t)t * W + c, n);
      };
      if constexpr (NS) {
#pragma unroll
        for (int t = 0; t < NS; ++t) one(t);
      } else {
        for (int t = 0; t < S; ++t) one(t);
      }
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      ss = fmaf(u[e], u[e], ss);
      u_row[c + e] = u[e];
    }
  }
  ss = block_sum(ss, scratch);
  const float inv = 1.f / sqrtf(ss / (float)W + a.eps);
  E* xn = reinterpret_cast<E*>(a.xn) + (size_t)row * W;
  for (int c = threadIdx.x * VEC; c < W; c += blockDim.x * VEC) {  // this thread's own u_row entries
    float v[VEC], w[VEC];
    ldn<VEC>(a.norm_w + c, w);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = u_row[c + e] * inv * w[e];
    stn<VEC>(xn + c, v);
  }
}

template <typename E, int VEC>
static void hyper_vec(const HyperArgs& a, hipStream_t st) {
  const int per = cdiv(a.W, VEC);
  // few rows: one row spread over up to 1024 threads (latency); many rows: 256 (several rows per CU)
  const int cap = a.T <= 256 ? 1024 : 256;
  const int block = std::min(cap, std::max(64, (per + 63) / 64 * 64));
  const size_t lds = (size_t)a.W * 4;
#define MLOP_HYPER(NS)                                                    \
  do {                                                                    \
    if (a.ids) hyper_kernel<E, NS, VEC, true><<<a.T, block, lds, st>>>(a);  \
    else hyper_kernel<E, NS, VEC, false><<<a.T, block, lds, st>>>(a);       \
  } while (0)
  switch (a.S) {
    case 1: MLOP_HYPER(1); break;
    case 2: MLOP_HYPER(2); break;
    case 3: MLOP_HYPER(3); break;
    case 4: MLOP_HYPER(4); break;
    case 6: MLOP_HYPER(6); break;
    case 8: MLOP_HYPER(8); break;
    default: MLOP_HYPER(0); break;
  }
#undef MLOP_HYPER
}

void launch_hyper(const HyperArgs& a, bool f32, hipStream_t st) {
  if (a.T == 0) return;
  if (f32) {
    if (a.W % 4 == 0) hyper_vec<float, 4>(a, st); else hyper_vec<float, 1>(a, st);
  } else {
    if (a.W % 4 == 0) hyper_vec<uint16_t, 4>(a, st); else hyper_vec<uint16_t, 1>(a, st);
  }
}

// an activation of columns n0 .. N of the rows, in place
template <typename E, int VEC>
__global__ void __launch_bounds__(256) act_columns_kernel(E* __restrict__ x, long total, int N, int n0, int act, float a, float b) {
  const long i = ((long)blockIdx.x * 256 + threadIdx.x) * VEC;
  if (i >= total) return;
  const int w = N - n0;
  E* p = x + i / w * N + n0 + i % w;
  float v[VEC];
  ldn<VEC>(p, v);
#pragma unroll
  for (int e = 0; e < VEC; ++e) {
    const float z = v[e];
    if (act == kActGelu) v[e] = z / (1.f + expf(-1.5957691216057308f * fmaf(0.044715f * z * z, z, z)));
    else if (act == kActXielu) v[e] = 0.5f * z + (z > 0.f ? a * z * z : b * (expm1f(z) - z));
    else v[e] = relu2_f(z);
  }
  stn<VEC>(p, v);
}

// out <- cap * tanh(x / cap), fp32
template <typename E, int VEC>
__global__ void __launch_bounds__(256) softcap_kernel(float* __restrict__ out, const E* __restrict__ x, long n,
                                                      float cap) {
  const long i = ((long)blockIdx.x * 256 + threadIdx.x) * VEC;
  if (i >= n) return;
  float v[VEC];
  ldn<VEC>(x + i, v);
#pragma unroll
  for (int e = 0; e < VEC; ++e) v[e] = cap * tanhf(v[e] / cap);
  stn<VEC>(out + i, v);
}

void launch_act_columns(void* x, long rows, int N, int n0, int act, float a, float b, bool f32, hipStream_t st) {
  const long total = rows * (N - n0);
  if (total == 0) return;
  const bool v8 = N % 8 == 0 && n0 % 8 == 0;
  const long grid = (total / (v8 ? 8 : 1) + 255) / 256;
  if (f32) {
    if (v8) act_columns_kernel<float, 8><<<grid, 256, 0, st>>>((float*)x, total, N, n0, act, a, b);
    else act_columns_kernel<float, 1><<<grid, 256, 0, st>>>((float*)x, total, N, n0, act, a, b);
  } else {
    if (v8) act_columns_kernel<uint16_t, 8><<<grid, 256, 0, st>>>((uint16_t*)x, total, N, n0, act, a, b);
    else act_columns_kernel<uint16_t, 1><<<grid, 256, 0, st>>>((uint16_t*)x, total, N, n0, act, a, b);
  }
}

void launch_softcap(float* out, const void* x, long n, float cap, bool f32, hipStream_t st) {
  if (n == 0) return;
  const bool v4 = n % 4 == 0;
  const long grid = (n / (v4 ? 4 : 1) + 255) / 256;
  if (f32) {
    if (v4) softcap_kernel<float, 4><<<grid, 256, 0, st>>>(out, (const float*)x, n, cap);
    else softcap_kernel<float, 1><<<grid, 256, 0, st>>>(out, (const float*)x, n, cap);
  } else {
    if (v4) softcap_kernel<uint16_t, 4><<<grid, 256, 0, st>>>(out, (const uint16_t*)x, n, cap);
    else softcap_kernel<uint16_t, 1><<<grid, 256, 0, st>>>(out, (const uint16_t*)x, n, cap);
  }
}

}  // namespace mlop
