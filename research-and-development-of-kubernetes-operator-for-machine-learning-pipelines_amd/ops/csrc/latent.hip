// Latent attention around attention_hd.hip's softmax: only a normed latent row c [R] per token is cached,
// and every head's keys and values are linear in it (k = U_k c, v = U_v c).
//
//   latent_store    the token's latent, RMS-normed, into its cache slot;
//   prompts         latent_gather copies the latents of a portion's keys (cached ones and its own) to one
//                   dense matrix, a GEMM expands them to keys and values, flash_hd reads those;
//   decode          head_mm takes the query to the latent space (q U_k per head), the paged kernel
//                   attends over latents as keys and as values, head_mm brings the result back (U_v per
//                   head, with the output gate), so a step reads each cached latent and no expansion.
#include "elem.h"
#include "mixers.h"

namespace mlop {

// a wave per token
template <typename E, int VEC>
__global__ void __launch_bounds__(256) latent_store_kernel(E* __restrict__ cache, const E* __restrict__ l, long ldl,
                                                           const float* __restrict__ w, float eps,
                                                           const int* __restrict__ slots, int T, int R, int RP) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (t >= T) return;
  const int slot = slots[t];
  if (slot < 0) return;
  const E* x = l + (size_t)t * ldl;
  float v[VEC], ss = 0.f;
  for (int c = lane * VEC; c < R; c += 64 * VEC) {
    ldn<VEC>(x + c, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) ss = fmaf(v[e], v[e], ss);
  }
  const float inv = 1.f / sqrtf(wave_sum(ss) / (float)R + eps);
  E* out = cache + (size_t)slot * RP;
  for (int c = lane * VEC; c < R; c += 64 * VEC) {
    float wv[VEC];
    ldn<VEC>(x + c, v);
    ldn<VEC>(w + c, wv);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] *= inv * wv[e];
    stn<VEC>(out + c, v);
  }
}

template <typename E>
static void latent_store_t(void* cache, const void* l, long ldl, const float* w, float eps, const int* slots, int T, int R,
                           int RP, hipStream_t st) {
  const bool al = ((reinterpret_cast<uintptr_t>(l) | reinterpret_cast<uintptr_t>(w)) & 15) == 0 && ldl % 8 == 0;
  const int grid = cdiv(T, 4);
  if (al && R % 8 == 0) latent_store_kernel<E, 8><<<grid, 256, 0, st>>>((E*)cache, (const E*)l, ldl, w, eps, slots, T, R, RP);
  else latent_store_kernel<E, 1><<<grid, 256, 0, st>>>((E*)cache, (const E*)l, ldl, w, eps, slots, T, R, RP);
}

void launch_latent_store(void* cache, const void* l, long ldl, const float* w, float eps, const int* slots, int T, int R,
                         int RP, int BS, bool f32, hipStream_t st) {
  (void)BS;  // one latent head: a slot is a row of the page array
  if (T == 0) return;
  if (f32) latent_store_t<float>(cache, l, ldl, w, eps, slots, T, R, RP, st);
  else latent_store_t<uint16_t>(cache, l, ldl, w, eps, slots, T, R, RP, st);
}

// 16 threads per row, 16 rows per workgroup; blockIdx.x = n_crows: the zero rows behind the last one
template <typename E>
__global__ void __launch_bounds__(256) latent_gather_kernel(LatentGatherArgs a) {
  constexpr int V = 16 / sizeof(E);
  const int sub = threadIdx.x & 15;
  const int i = blockIdx.y * 16 + (threadIdx.x >> 4);
  E* out = reinterpret_cast<E*>(a.out);
  if ((int)blockIdx.x == a.n_crows) {
    if (i >= a.pad) return;
    for (int c = sub * V; c < a.RP; c += 16 * V)
      *reinterpret_cast<u32x4*>(out + (size_t)(a.rows + i) * a.RP + c) = u32x4{0, 0, 0, 0};
    return;
  }
  const int s = a.crow_seq[blockIdx.x], ctx = a.ctx_len[s];
  const int pos = key_region_start(ctx - a.q_len[s], a.window) + i;
  if (pos >= ctx) return;
  const long row = (long)a.xbase[s] + pos;
  if (row < 0 || row >= a.rows) return;
  const int page = min(max(a.bt[(size_t)s * a.bt_stride + pos / a.BS], 0), a.num_blocks - 1);
  const E* src = reinterpret_cast<const E*>(a.cache) + ((size_t)page * a.BS + pos % a.BS) * a.RP;
  for (int c = sub * V; c < a.RP; c += 16 * V)
    *reinterpret_cast<u32x4*>(out + (size_t)row * a.RP + c) = *reinterpret_cast<const u32x4*>(src + c);
}

void launch_latent_gather(const LatentGatherArgs& a, bool f32, hipStream_t st) {
  const dim3 grid(a.n_crows + 1, cdiv(a.x_max > a.pad ? a.x_max : a.pad, 16));
  if (f32) latent_gather_kernel<float><<<grid, 256, 0, st>>>(a);
  else latent_gather_kernel<uint16_t><<<grid, 256, 0, st>>>(a);
}

namespace {

__device__ __forceinline__ int tile_token(const HeadMmArgs& a, int i) { return a.q_start[a.tile_seq[i]] + a.tile_q0[i]; }
__device__ __forceinline__ float gate_f(float g) { return 1.f / (1.f + __expf(-g)); }

}  // namespace

// A workgroup: one head, 64 NT output columns (16 NT per wave), 16 MT tiles.
template <int MT, int NT>
__global__ void __launch_bounds__(256) head_mm_kernel(HeadMmArgs a) {
  const int h = blockIdx.x, lane = threadIdx.x & 63, wid = threadIdx.x >> 6, l15 = lane & 15, g4 = lane >> 4;
  const int n0 = (blockIdx.y * 4 + wid) * 16 * NT, m0 = blockIdx.z * 16 * MT;
  if (n0 >= a.N) return;
  const uint16_t* w[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n)
    w[n] = reinterpret_cast<const uint16_t*>(a.w) + ((size_t)h * a.N + min(n0 + 16 * n + l15, a.N - 1)) * a.K + 8 * g4;
  const uint16_t* x[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int i = min(m0 + 16 * m + l15, a.n_tiles - 1);
    x[m] = reinterpret_cast<const uint16_t*>(a.x) + (size_t)(a.x_tok ? tile_token(a, i) : i) * a.ldx + h * a.hx + 8 * g4;
  }
  f32x4 acc[MT][NT];
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int n = 0; n < NT; ++n) acc[m][n] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k = 0; k < a.K; k += 64) {
    bf16x8 wf[2][NT], xf[2][MT];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
#pragma unroll
      for (int n = 0; n < NT; ++n) wf[u][n] = *reinterpret_cast<const bf16x8*>(w[n] + k + 32 * u);
#pragma unroll
      for (int m = 0; m < MT; ++m) xf[u][m] = *reinterpret_cast<const bf16x8*>(x[m] + k + 32 * u);
    }
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int n = 0; n < NT; ++n) acc[m][n] = mfma16(wf[u][n], xf[u][m], acc[m][n]);
  }
  // row 4 g4 + e of a product = output column, column l15 = tile
  const bool vec = a.N % 4 == 0 && (a.ldo | a.ho) % 4 == 0 && (!a.gate || a.ldg % 4 == 0);
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int i = m0 + 16 * m + l15;
    if (i >= a.n_tiles) continue;
    const int tok = a.out_tok || a.gate ? tile_token(a, i) : 0;
    const uint16_t* gate = reinterpret_cast<const uint16_t*>(a.gate) + (size_t)tok * a.ldg + (size_t)h * a.N;
    uint16_t* out = reinterpret_cast<uint16_t*>(a.out) + (size_t)(a.out_tok ? tok : i) * a.ldo + h * a.ho;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int n = n0 + 16 * t + 4 * g4;
      if (n >= a.N) continue;
      float v[4] = {acc[m][t][0], acc[m][t][1], acc[m][t][2], acc[m][t][3]};
      if (vec) {
        if (a.gate) {
          float g[4];
          ldn<4>(gate + n, g);
#pragma unroll
          for (int e = 0; e < 4; ++e) v[e] *= gate_f(g[e]);
        }
        stn<4>(out + n, v);
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (n + e < a.N) out[n + e] = f2bf(a.gate ? v[e] * gate_f(bf2f(gate[n + e])) : v[e]);
      }
    }
  }
}

// plain form (fp32): one thread per output
__global__ void __launch_bounds__(256) head_mm_plain_kernel(HeadMmArgs a) {
  const int h = blockIdx.x, n = blockIdx.y * 256 + threadIdx.x, i = blockIdx.z;
  if (n >= a.N) return;
  const int tok = tile_token(a, i);
  const float* x = reinterpret_cast<const float*>(a.x) + (size_t)(a.x_tok ? tok : i) * a.ldx + h * a.hx;
  const float* w = reinterpret_cast<const float*>(a.w) + ((size_t)h * a.N + n) * a.K;
  float v = 0.f;
  for (int k = 0; k < a.K; ++k) v = fmaf(x[k], w[k], v);
  if (a.gate) v /= 1.f + expf(-reinterpret_cast<const float*>(a.gate)[(size_t)tok * a.ldg + (size_t)h * a.N + n]);
  reinterpret_cast<float*>(a.out)[(size_t)(a.out_tok ? tok : i) * a.ldo + h * a.ho + n] = v;
}

void launch_head_mm(const HeadMmArgs& a, bool f32, hipStream_t st) {
  if (a.n_tiles == 0) return;
  if (f32) {
    head_mm_plain_kernel<<<dim3(a.H, cdiv(a.N, 256), a.n_tiles), 256, 0, st>>>(a);
  } else if (a.n_tiles > 64) {
    head_mm_kernel<4, 2><<<dim3(a.H, cdiv(a.N, 128), cdiv(a.n_tiles, 64)), 256, 0, st>>>(a);
  } else if (a.n_tiles > 16) {
    head_mm_kernel<2, 1><<<dim3(a.H, cdiv(a.N, 64), cdiv(a.n_tiles, 32)), 256, 0, st>>>(a);
  } else {
    head_mm_kernel<1, 1><<<dim3(a.H, cdiv(a.N, 64), 1), 256, 0, st>>>(a);
  }
}

}  // namespace mlop
