// Latent attention around attention_hd.hip's softmax: only a normed latent row c [R] per token is cached,
// and every head's keys and values are linear in it (k = U_k c, v = U_v c).
//
//   latent_store    the token's latent, RMS-normed, into its cache slot, a key part shared by all heads,
//                   turned by the position, behind it; the queries' latent is normed beside them;
//   prompts         latent_gather copies the latents of a portion's keys (cached ones and its own) to one
//                   dense matrix, a GEMM expands them to keys and values, flash_hd reads those;
//   decode          head_mm takes the query to the latent space (q U_k per head), the paged kernel
//                   attends over latents as keys and as values, head_mm brings the result back (U_v per
//                   head, with the output gate), so a step reads each cached latent and no expansion.
#include "elem.h"
#include "mixers.h"

namespace mlop {

// the pair (u, v) turned by position p; n: rotated dims
__device__ __forceinline__ void turn(const float* table, int p, int n_pos, int n, int pair, float& u, float& v) {
  const float* cs = table + (size_t)min(max(p, 0), n_pos - 1) * n + pair;
  const float c = cs[0], s = cs[n >> 1], x = u;
  u = x * c - v * s;
  v = v * c + x * s;
}

// one wave: out = w * x / rms(x), zeros from n to n_pad
template <typename E, int VEC>
__device__ __forceinline__ void norm_row(E* out, const E* x, const float* w, int n, int n_pad, float eps, int lane) {
  float v[VEC], ss = 0.f;
  for (int c = lane * VEC; c < n; c += 64 * VEC) {
    ldn<VEC>(x + c, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) ss = fmaf(v[e], v[e], ss);
  }
  const float inv = 1.f / sqrtf(wave_sum(ss) / (float)n + eps);
  for (int c = lane * VEC; c < n_pad; c += 64 * VEC) {
    float wv[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = 0.f;
    if (c < n) {
      ldn<VEC>(x + c, v);
      ldn<VEC>(w + c, wv);
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] *= inv * wv[e];
    }
    stn<VEC>(out + c, v);
  }
}

// a wave per token and job (its latent and rotated key; its query latent)
template <typename E, int VEC>
__global__ void __launch_bounds__(256) latent_store_kernel(LatentStoreArgs a) {
  const int lane = threadIdx.x & 63, jobs = (a.l ? 1 : 0) + (a.q ? 1 : 0);
  const int unit = blockIdx.x * 4 + (threadIdx.x >> 6), t = unit / jobs;
  if (t >= a.T) return;
  if (!a.l || unit % jobs) {
    norm_row<E, VEC>(reinterpret_cast<E*>(a.q_out) + (size_t)t * a.QP, reinterpret_cast<const E*>(a.q) + (size_t)t * a.ldq,
                     a.q_w, a.QR, a.QP, a.eps, lane);
    return;
  }
  const int slot = a.slots[t];
  if (slot < 0) return;
  E* row = reinterpret_cast<E*>(a.cache) + (size_t)slot * a.RP;
  if (a.k) {
    const E* k = reinterpret_cast<const E*>(a.k) + (size_t)t * a.ldk;
    const int p = a.pos[t];
    for (int i = lane; i < a.n_rot >> 1; i += 64) {
      float u = ld1(k + 2 * i), v = ld1(k + 2 * i + 1);
      turn(a.table, p, a.n_pos, a.n_rot, i, u, v);
      st1(row + a.off + 2 * i, u);
      st1(row + a.off + 2 * i + 1, v);
    }
  }
  norm_row<E, VEC>(row, reinterpret_cast<const E*>(a.l) + (size_t)t * a.ldl, a.w, a.R, a.R, a.eps, lane);
}

template <typename E>
static void latent_store_t(const LatentStoreArgs& a, hipStream_t st) {
  auto al = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  const bool v8 = (!a.l || (al(a.l) && al(a.w) && a.ldl % 8 == 0 && a.R % 8 == 0)) &&
                  (!a.q || (al(a.q) && al(a.q_w) && a.ldq % 8 == 0 && a.QR % 8 == 0 && a.QP % 8 == 0));
  const int grid = cdiv(a.T * ((a.l ? 1 : 0) + (a.q ? 1 : 0)), 4);
  if (v8) latent_store_kernel<E, 8><<<grid, 256, 0, st>>>(a);
  else latent_store_kernel<E, 1><<<grid, 256, 0, st>>>(a);
}

void launch_latent_store(const LatentStoreArgs& a, bool f32, hipStream_t st) {
  if (a.T == 0 || (!a.l && !a.q)) return;
  if (f32) latent_store_t<float>(a, st);
  else latent_store_t<uint16_t>(a, st);
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

// the columns behind a head's products: the rotated query part, then zeros (n tiles from m0)
template <typename E>
__device__ __forceinline__ void head_rot(const HeadMmArgs& a, int h, int m0, int n) {
  const int pairs = a.extra >> 1;
  for (int x = threadIdx.x; x < n * pairs; x += 256) {
    const int i = m0 + x / pairs, p = x % pairs;
    if (i >= a.n_tiles) return;
    const int tok = tile_token(a, i);
    float u = 0.f, v = 0.f;
    if (2 * p < a.n_rot) {
      const E* src = reinterpret_cast<const E*>(a.x) + (size_t)(a.x_tok ? tok : i) * a.ldx + h * a.hx + a.x_off + 2 * p;
      u = ld1(src), v = ld1(src + 1);
      turn(a.table, a.pos[tok], a.n_pos, a.n_rot, p, u, v);
    }
    E* out = reinterpret_cast<E*>(a.out) + (size_t)(a.out_tok ? tok : i) * a.ldo + h * a.ho + a.N + 2 * p;
    st1(out, u);
    st1(out + 1, v);
  }
}

// A workgroup: one head, 64 NT output columns (16 NT per wave), 16 MT tiles; with a table, the last of a
// head's workgroups has the columns behind the products.
template <int MT, int NT>
__global__ void __launch_bounds__(256) head_mm_kernel(HeadMmArgs a) {
  const int h = blockIdx.x, lane = threadIdx.x & 63, wid = threadIdx.x >> 6, l15 = lane & 15, g4 = lane >> 4;
  const int n0 = (blockIdx.y * 4 + wid) * 16 * NT, m0 = blockIdx.z * 16 * MT;
  if (a.table && blockIdx.y == gridDim.y - 1) return head_rot<uint16_t>(a, h, m0, 16 * MT);
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
  if (a.table && blockIdx.y == gridDim.y - 1) return head_rot<float>(a, h, i, 1);
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
  const int more = a.table ? 1 : 0;
  if (f32) {
    head_mm_plain_kernel<<<dim3(a.H, cdiv(a.N, 256) + more, a.n_tiles), 256, 0, st>>>(a);
  } else if (a.n_tiles > 64) {
    head_mm_kernel<4, 2><<<dim3(a.H, cdiv(a.N, 128) + more, cdiv(a.n_tiles, 64)), 256, 0, st>>>(a);
  } else if (a.n_tiles > 16) {
    head_mm_kernel<2, 1><<<dim3(a.H, cdiv(a.N, 64) + more, cdiv(a.n_tiles, 32)), 256, 0, st>>>(a);
  } else {
    head_mm_kernel<1, 1><<<dim3(a.H, cdiv(a.N, 64) + more, 1), 256, 0, st>>>(a);
  }
}

}  // namespace mlop
