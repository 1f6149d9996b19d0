// The fp32 residual stream of a decoder with a norm before and behind every sublayer, and two
// elementwise steps such decoders use:
//
//   residual    x <- x + post_w * y / rms(y)   (or x + y),   xn = norm_w * x / rms(x)   (or x)
//               where y may be a token's expert rows summed (weighted, with the token's own input as one of
//               them), beside a gated shared row; or xn = norm_w * tanh(alpha x) + b (dynamic tanh: no statistics)
//   gated norm  group norm of y with a gate before or behind it
//   clamp_glu   clamped gated unit of a feed-forward's [gate | up] columns
//
// A row's elements stay in registers between its sums of squares and the stores, so each pass reads
// and writes every operand once (HBM-bound).
#include <algorithm>
#include <type_traits>

#include "elem.h"
#include "mixers.h"

namespace mlop {

enum { kStart = 0, kStep = 1, kExperts = 2 };  // residual_kernel: where y comes from

template <typename E, int VEC, int NI, int KIND>
__global__ void __launch_bounds__(1024) residual_kernel(ResidualArgs a) {
  __shared__ float scratch[16];
  constexpr bool START = KIND == kStart;
  const int row = blockIdx.x, W = a.W, tid = threadIdx.x, BT = blockDim.x;
  const float post1 = a.post_one ? *a.post_w : 1.f, norm1 = a.norm_one ? *a.norm_w : 1.f;
  float* xr = a.x + (size_t)row * W;
  float x[NI][VEC], y[NI][VEC], pw[NI][VEC], nw[NI][VEC];
  const E* yr;
  const E* pr = nullptr;
  if constexpr (START) {
    yr = reinterpret_cast<const E*>(a.table) + (size_t)min(max(a.ids[row], 0l), a.vocab - 1) * W;
    if (a.pos_table) pr = reinterpret_cast<const E*>(a.pos_table) + (size_t)min((long)max(a.pos[row], 0), a.n_pos - 1) * W;
  } else {
    yr = reinterpret_cast<const E*>(a.y) + (a.y ? (size_t)row * W : 0);
  }
  const bool post_v = a.post_w && !a.post_one, norm_v = a.norm_w && !a.norm_one;
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = (tid + BT * i) * VEC;
    if (c < W) {
#pragma unroll
      for (int e = 0; e < VEC; ++e) pw[i][e] = post1, nw[i][e] = norm1, y[i][e] = 0.f;
      if (KIND != kExperts || a.y) ldn<VEC>(yr + c, y[i]);
      if (KIND != kExperts && norm_v) ldn<VEC>(a.norm_w + c, nw[i]);
      if constexpr (START) {
        float p[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) p[e] = 0.f;
        if (pr) ldn<VEC>(pr + c, p);
#pragma unroll
        for (int e = 0; e < VEC; ++e) x[i][e] = fmaf(a.embed_scale, y[i][e], p[e]);
      } else {
        ldn<VEC>(xr + c, x[i]);
        if (KIND != kExperts && post_v) ldn<VEC>(a.post_w + c, pw[i]);
      }
    }
  }
  if constexpr (KIND == kExperts) {
    if (a.gate) {
      const float g = a.gate[row];
#pragma unroll
      for (int i = 0; i < NI; ++i)
#pragma unroll
        for (int e = 0; e < VEC; ++e) y[i][e] *= g;
    }
    const int* inv = a.inv + (size_t)row * a.top;
    const float* row_w = a.row_w + (a.row_w ? (size_t)row * a.top : 0);
    const E* self = reinterpret_cast<const E*>(a.self) + (a.self ? (size_t)row * W : 0);
    const E* none = a.y ? yr : reinterpret_cast<const E*>(a.rows);  // read with weight 0 where there is no row
    const int total = a.top + (a.self != nullptr);
    // N rows at a time, all of them in flight before the first is added
    auto add = [&](int j0, auto n_) {
      constexpr int N = decltype(n_)::value;
      struct alignas(sizeof(E) * VEC) Pack {
        E e[VEC];
      };
      const E* er[N];
      float w[N];
      Pack v[N][NI];
#pragma unroll
      for (int k = 0; k < N; ++k) {
        const int j = j0 + k, r = j < a.top ? inv[j] : -1;
        er[k] = r >= 0 ? reinterpret_cast<const E*>(a.rows) + (size_t)r * W : none;
        w[k] = r < 0 ? 0.f : a.row_w ? row_w[j] : 1.f;
        if (j == a.top && a.self) er[k] = self, w[k] = a.self_w[row];
      }
#pragma unroll
      for (int k = 0; k < N; ++k)
#pragma unroll
        for (int i = 0; i < NI; ++i) {
          const int c = (tid + BT * i) * VEC;
          v[k][i] = *reinterpret_cast<const Pack*>(er[k] + (c < W ? c : 0));
        }
#pragma unroll
      for (int k = 0; k < N; ++k)
#pragma unroll
        for (int i = 0; i < NI; ++i)
#pragma unroll
          for (int e = 0; e < VEC; ++e) y[i][e] = fmaf(w[k], w[k] != 0.f ? ld1(&v[k][i].e[e]) : 0.f, y[i][e]);
    };
    int j = 0;
    if (total != 2)
      for (; j + 2 < total; j += 4) add(j, std::integral_constant<int, 4>{});
    for (; j < total; j += 2) add(j, std::integral_constant<int, 2>{});
    // (behind the rows: registers)
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (tid + BT * i) * VEC;
      if (c < W) {
        if (norm_v) ldn<VEC>(a.norm_w + c, nw[i]);
        if (post_v) ldn<VEC>(a.post_w + c, pw[i]);
      }
    }
  }
  if constexpr (!START) {
    float inv = 1.f;
    if (a.post_w) {
#pragma unroll
      for (int i = 0; i < NI; ++i)
        if ((tid + BT * i) * VEC < W) {
#pragma unroll
          for (int e = 0; e < VEC; ++e) ss = fmaf(y[i][e], y[i][e], ss);
        }
      inv = 1.f / sqrtf(block_sum(ss, scratch) / (float)a.n + a.eps);
    }
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
      for (int e = 0; e < VEC; ++e) x[i][e] += a.post_w ? y[i][e] * inv * pw[i][e] : y[i][e];
  }
  ss = 0.f;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = (tid + BT * i) * VEC;
    if (c < W) {
      if (a.store) stn<VEC>(xr + c, x[i]);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss = fmaf(x[i][e], x[i][e], ss);
    }
  }
  E* xn = reinterpret_cast<E*>(a.xn) + (size_t)row * W;
  if (a.tanh_a) {
    const float alpha = *a.tanh_a;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (tid + BT * i) * VEC;
      if (c < W) {
        float nb[VEC];
        ldn<VEC>(a.tanh_b + c, nb);
#pragma unroll
        for (int e = 0; e < VEC; ++e) x[i][e] = fmaf(tanh_f(alpha * x[i][e]), nw[i][e], nb[e]);
        stn<VEC>(xn + c, x[i]);
      }
    }
    return;
  }
  const float inv = a.norm_w ? 1.f / sqrtf(block_sum(ss, scratch) / (float)a.n + a.eps) : 1.f;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = (tid + BT * i) * VEC;
    if (c < W) {
#pragma unroll
      for (int e = 0; e < VEC; ++e) x[i][e] *= inv * nw[i][e];
      stn<VEC>(xn + c, x[i]);
    }
  }
}

template <typename E, int VEC, int NI>
static void residual_ni(const ResidualArgs& a, int block, hipStream_t st) {
  if (a.ids) residual_kernel<E, VEC, NI, kStart><<<a.T, block, 0, st>>>(a);
  else if (a.rows) residual_kernel<E, VEC, NI, kExperts><<<a.T, block, 0, st>>>(a);
  else residual_kernel<E, VEC, NI, kStep><<<a.T, block, 0, st>>>(a);
}

template <typename E, int VEC>
static void residual_vec(const ResidualArgs& a, hipStream_t st) {
  const int per = cdiv(a.W, VEC);
  // few rows: a row over up to 1024 threads (latency); many: 256 (several rows per CU)
  int ni = a.T <= 256 ? 1 : std::min(a.rows ? 2 : 4, cdiv(per, 256));
  if (cdiv(per, ni) > 1024) ni = cdiv(per, 1024);
  const int p2 = ni <= 1 ? 1 : ni <= 2 ? 2 : ni <= 4 ? 4 : 16;
  const int block = cdiv(cdiv(per, p2), 64) * 64;
  if (p2 == 1) residual_ni<E, VEC, 1>(a, block, st);
  else if (p2 == 2) residual_ni<E, VEC, 2>(a, block, st);
  else if (p2 == 4) residual_ni<E, VEC, 4>(a, block, st);
  else if constexpr (VEC == 1) residual_ni<E, VEC, 16>(a, block, st);
}

void launch_residual(const ResidualArgs& a, bool f32, hipStream_t st) {
  if (a.T == 0) return;
  if (f32) {
    if (a.W % 4 == 0) residual_vec<float, 4>(a, st); else residual_vec<float, 1>(a, st);
  } else {
    if (a.W % 4 == 0) residual_vec<uint16_t, 4>(a, st); else residual_vec<uint16_t, 1>(a, st);
  }
}

__device__ __forceinline__ float sigmoid_f(float x) { return __builtin_amdgcn_rcpf(1.f + __expf(-x)); }

// BT threads (16, 64 or 256) per (token, group); NI > 0: the group's values stay in registers, 0: they are
// read twice
template <typename E, int VEC, int BT, int NI>
__global__ void __launch_bounds__(256) gated_norm_kernel(GatedNormArgs a) {
  __shared__ float scratch[16];
  constexpr int N = NI ? NI : 1;
  const int gw = a.n / a.groups;
  const long unit = (long)blockIdx.x * (256 / BT) + threadIdx.x / BT;
  if (unit >= (long)a.T * a.groups) return;  // whole groups of BT threads, and no barrier below when BT < 256
  const int t = (int)(unit / a.groups), g = (int)(unit % a.groups), tid = threadIdx.x % BT;
  const E* y = reinterpret_cast<const E*>(a.y) + (size_t)t * a.n + (size_t)g * gw;
  const E* gt = reinterpret_cast<const E*>(a.gate) + (size_t)t * a.ldg + (size_t)g * gw;
  const float* w = a.w + (size_t)g * gw;
  E* out = reinterpret_cast<E*>(a.out) + (size_t)t * a.n + (size_t)g * gw;
  auto act = [&](float z) { return a.act == kGateSilu ? z * sigmoid_f(z) : sigmoid_f(z); };
  float v[N][VEC], z[N][VEC];
  auto load = [&](int c, float (&vv)[VEC], float (&zz)[VEC]) {
    ldn<VEC>(y + c, vv);
    ldn<VEC>(gt + c, zz);
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      zz[e] = act(zz[e]);
      if (a.gate_first) vv[e] *= zz[e];
    }
  };
  float ss = 0.f;
  if constexpr (NI > 0) {
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (tid + BT * i) * VEC;
      if (c < gw) {
        load(c, v[i], z[i]);
#pragma unroll
        for (int e = 0; e < VEC; ++e) ss = fmaf(v[i][e], v[i][e], ss);
      }
    }
  } else {
    for (int c = tid * VEC; c < gw; c += BT * VEC) {
      load(c, v[0], z[0]);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss = fmaf(v[0][e], v[0][e], ss);
    }
  }
  if constexpr (BT == 16) {
    ss += detail::dpp<0xB1>(ss);
    ss += detail::dpp<0x4E>(ss);
    ss += detail::dpp<0x141>(ss);
    ss += detail::dpp<0x140>(ss);
  } else {
    ss = BT == 64 ? wave_sum(ss) : block_sum(ss, scratch);
  }
  const float inv = 1.f / sqrtf(ss / (float)gw + a.eps);
  auto put = [&](int c, float (&vv)[VEC], float (&zz)[VEC]) {
    float wv[VEC];
    ldn<VEC>(w + c, wv);
#pragma unroll
    for (int e = 0; e < VEC; ++e) vv[e] = vv[e] * inv * wv[e] * (a.gate_first ? 1.f : zz[e]);
    stn<VEC>(out + c, vv);
  };
  if constexpr (NI > 0) {
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (tid + BT * i) * VEC;
      if (c < gw) put(c, v[i], z[i]);
    }
  } else {
    for (int c = tid * VEC; c < gw; c += BT * VEC) {
      load(c, v[0], z[0]);
      put(c, v[0], z[0]);
    }
  }
}

template <typename E, int VEC>
static void gated_norm_vec(const GatedNormArgs& a, hipStream_t st) {
  const int gw = a.n / a.groups;
  const long units = (long)a.T * a.groups;
#define MLOP_GN(BT, NI) gated_norm_kernel<E, VEC, BT, NI><<<(int)((units * BT + 255) / 256), 256, 0, st>>>(a)
  if (gw <= 16 * VEC) MLOP_GN(16, 1);
  else if (gw <= 32 * VEC) MLOP_GN(16, 2);
  else if (gw <= 64 * VEC) MLOP_GN(64, 1);
  else if (gw <= 128 * VEC) MLOP_GN(64, 2);
  else if (gw <= 256 * VEC) MLOP_GN(256, 1);
  else if (gw <= 1024 * VEC) MLOP_GN(256, 4);
  else MLOP_GN(256, 0);
#undef MLOP_GN
}

void launch_gated_norm(const GatedNormArgs& a, bool f32, hipStream_t st) {
  if (a.T == 0) return;
  const int gw = a.n / a.groups;
  const bool al = ((reinterpret_cast<uintptr_t>(a.gate) | reinterpret_cast<uintptr_t>(a.y) |
                    reinterpret_cast<uintptr_t>(a.out) | reinterpret_cast<uintptr_t>(a.w)) & 15) == 0;
  const bool v4 = al && gw % 4 == 0 && a.ldg % 8 == 0, v8 = v4 && gw % 8 == 0;
  if (f32) {
    if (v4) gated_norm_vec<float, 4>(a, st); else gated_norm_vec<float, 1>(a, st);
  } else {
    if (v8) gated_norm_vec<uint16_t, 8>(a, st);
    else if (v4) gated_norm_vec<uint16_t, 4>(a, st);
    else gated_norm_vec<uint16_t, 1>(a, st);
  }
}

// x [T, 2 I], gate and up columns interleaved in groups of 16 (the GEMM epilogue's layout)
template <typename E>
__global__ void __launch_bounds__(256) clamp_glu_kernel(E* __restrict__ out, const E* __restrict__ x, long total, int I,
                                                        float alpha, float limit) {
  for (long v = blockIdx.x * 256l + threadIdx.x; v < total; v += (long)gridDim.x * 256) {
    const long t = v / (I / 4);
    const int c = (int)(v % (I / 4)) * 4;
    const E* row = x + t * 2 * I + (c / 16) * 32 + c % 16;
    float g[4], u[4];
    ldn<4>(row, g);
    ldn<4>(row + 16, u);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      if (alpha > 0.f) {  // (in fp32 to the last bits: an exact quotient)
        const float z = fminf(g[e], limit), up = fminf(fmaxf(u[e], -limit), limit);
        g[e] = z * (up + 1.f) / (1.f + expf(-alpha * z));
      } else {
        g[e] = g[e] / (1.f + expf(-g[e])) * u[e];
      }
    }
    stn<4>(out + t * I + c, g);
  }
}

void launch_clamp_glu(void* out, const void* x, int T, int I, float alpha, float limit, bool f32, hipStream_t st) {
  if (T == 0) return;
  const long total = (long)T * (I / 4);
  const int grid = (int)std::min<long>((total + 255) / 256, 8192);
  if (f32) clamp_glu_kernel<float><<<grid, 256, 0, st>>>((float*)out, (const float*)x, total, I, alpha, limit);
  else clamp_glu_kernel<uint16_t><<<grid, 256, 0, st>>>((uint16_t*)out, (const uint16_t*)x, total, I, alpha, limit);
}

}  // namespace mlop
