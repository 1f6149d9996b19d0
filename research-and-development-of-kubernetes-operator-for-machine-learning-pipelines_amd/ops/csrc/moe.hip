// Mixture-of-experts routing kernels for gfx950 (K11 route, K12 permute, K14 combine).
// The expert FFN itself is the grouped MFMA GEMM of gemm.hip (K13).
//
// Three kinds of routing:
//   kSoftmax  softmax over the router's logits, renormalised over the chosen experts, the weights on the experts'
//             outputs (moe_combine);
//   kSigmoid  fp32 logits, the chosen experts' sigmoid scores as they are, the scores on the experts' INPUT rows, and
//             possibly one row behind the experts' whose sigmoid is a gate per token;
//   kGroups   fp32 logits, softmax over all of them, scores as they are on the experts' outputs (residual.hip sums
//             them); a correction per output and a choice of groups decide who is chosen; outputs behind the experts'
//             are identity experts, which have no row.
//
// Everything stays on the device and has static shapes (T*k rows reserved, the
// valid count lives in offsets[n_local]), so an MoE layer can be captured in
// a hipGraph: no host sync to size the permuted batch.
//
// Combine is a deterministic gather (out[t] = sum_j w[t,j] * y[inv[t*k+j]],
// fp32 accumulate, one bf16 rounding), not an atomic scatter: bitwise
// reproducible whatever order the permutation assigned rows in
// (cdna_hip_programming.md App. B "Scatter / gather": store-then-sum form).
#include <stdexcept>

#include "common.h"
#include "launch.h"

namespace mlop {

// one thread per token: softmax over E router logits (bf16 in), top-k, renormalise
__global__ void moe_route_kernel(float* __restrict__ topw, int* __restrict__ topi,
                                 const uint16_t* __restrict__ logits, int T, int E, int k) {
  const int t = blockIdx.x * blockDim.x + threadIdx.x;
  if (t >= T) return;
  const uint16_t* l = logits + (size_t)t * E;
  float v[64];
  float mx = -INFINITY;
  for (int e = 0; e < E; ++e) {
    v[e] = bf2f(l[e]);
    mx = fmaxf(mx, v[e]);
  }
  float s = 0.f;
  for (int e = 0; e < E; ++e) {
    v[e] = __expf(v[e] - mx);
    s += v[e];
  }
  const float inv = 1.f / s;
  float picked = 0.f;
  unsigned long long used = 0ull;
  for (int j = 0; j < k; ++j) {
    int best = 0;
    float bv = -1.f;
    for (int e = 0; e < E; ++e)
      if (!((used >> e) & 1ull) && v[e] > bv) { bv = v[e]; best = e; }
    used |= 1ull << best;
    topi[t * k + j] = best;
    topw[t * k + j] = bv * inv;
    picked += bv * inv;
  }
  const float rn = picked > 0.f ? 1.f / picked : 0.f;
  for (int j = 0; j < k; ++j) topw[t * k + j] *= rn;
}

// counting sort of the T*k routed slots by local expert (one workgroup)
__global__ void __launch_bounds__(1024) moe_sort_kernel(int* __restrict__ offsets,
                                                       int* __restrict__ src,
                                                       int* __restrict__ inv,
                                                       const int* __restrict__ topi, int n_slots,
                                                       int e0, int n_local) {
  __shared__ int cnt[256];
  __shared__ int base[257];
  for (int e = threadIdx.x; e < n_local; e += blockDim.x) cnt[e] = 0;
  __syncthreads();
  for (int s = threadIdx.x; s < n_slots; s += blockDim.x) {
    const int e = topi[s] - e0;
    inv[s] = (e >= 0 && e < n_local) ? atomicAdd(&cnt[e], 1) : -1;
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    int acc = 0;
    for (int e = 0; e < n_local; ++e) {
      base[e] = acc;
      offsets[e] = acc;
      acc += cnt[e];
    }
    base[n_local] = acc;
    offsets[n_local] = acc;
  }
  __syncthreads();
  for (int s = threadIdx.x; s < n_slots; s += blockDim.x) {
    const int e = topi[s] - e0;
    if (e >= 0 && e < n_local) {
      const int row = base[e] + inv[s];
      inv[s] = row;
      src[row] = s;
    }
  }
}

// xp[r] = x[src[r] / k] for the valid rows (one workgroup per row)
__global__ void __launch_bounds__(256) moe_gather_kernel(uint16_t* __restrict__ xp,
                                                        const uint16_t* __restrict__ x,
                                                        const int* __restrict__ src,
                                                        const int* __restrict__ offsets,
                                                        int n_local, int k, int H) {
  const int r = blockIdx.x;
  if (r >= offsets[n_local]) return;
  const int t = src[r] / k;
  const uint16_t* a = x + (size_t)t * H;
  uint16_t* b = xp + (size_t)r * H;
  for (int c = threadIdx.x * 8; c < H; c += blockDim.x * 8)
    *reinterpret_cast<u32x4*>(b + c) = *reinterpret_cast<const u32x4*>(a + c);
}

// out[t] = sum_j topw[t, j] * y[inv[t*k + j]]   (slots with inv < 0 are not local: skipped)
__global__ void __launch_bounds__(256) moe_combine_kernel(uint16_t* __restrict__ out,
                                                         const uint16_t* __restrict__ y,
                                                         const int* __restrict__ inv,
                                                         const float* __restrict__ topw, int k,
                                                         int H) {
  const int t = blockIdx.x;
  for (int c = threadIdx.x * 8; c < H; c += blockDim.x * 8) {
    float acc[8] = {0, 0, 0, 0, 0, 0, 0, 0};
    for (int j = 0; j < k; ++j) {
      const int r = inv[t * k + j];
      if (r < 0) continue;
      const float w = topw[t * k + j];
      u32x4 v = *reinterpret_cast<const u32x4*>(y + (size_t)r * H + c);
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        acc[2 * q] += w * lo_bf(v[q]);
        acc[2 * q + 1] += w * hi_bf(v[q]);
      }
    }
    u32x4 o;
#pragma unroll
    for (int q = 0; q < 4; ++q) o[q] = pack2(acc[2 * q], acc[2 * q + 1]);
    *reinterpret_cast<u32x4*>(out + (size_t)t * H + c) = o;
  }
}

// ---------------------------------------------------------------------------
// Optional prologue (MoePro): the post-attention residual add + RMSNorm that produces x, so
// the O projection's output goes straight into the MoE block (one more launch saved).
struct MoePro {
  const uint16_t* y;   // [T, H] O projection output (nullptr: no prologue, x given)
  uint16_t* residual;  // [T, H] in / out
  const uint16_t* w;   // [H] post-attention norm weight
  float eps;
  uint16_t* xn;        // [T, H] normed x (written)
};

// Decode-size MoE dispatch in ONE launch (T <= kSmallT tokens): router GEMV (bf16-rounded
// logits, as the separate router projection stores them), softmax / top-k / renormalise,
// counting sort by local expert and the row gather.  At batch 1-16 each of the four
// separate launches (router GEMV, route, sort, gather) is a ~5 us graph node doing <1 us of
// work (profiles/r02_mixtral_b1.md); one workgroup does all four back to back.
// Wave w computes the logits of experts w, w+8, ...: the expert's router row is loaded once
// (all of a lane's chunks in flight together) while the wave walks the T activation rows.
constexpr int kSmallT = 16, kMaxE = 64, kDispWaves = 8;

enum { kSoftmax = 0, kSigmoid = 1, kGroups = 2 };

// kSigmoid: `rows` router rows, the first E of them experts'
struct SigArgs {
  float* gate;   // [T] sigmoid of row E (nullptr: there is none)
  float* row_w;  // [T * k] score of each permuted row (the gathered rows hold it already: nullptr)
  int rows;
};
__device__ __forceinline__ float sigmoid_of(float z) { return 1.f / (1.f + __expf(-z)); }

// the largest of n logits behind (v, i) in the order of falling value, then rising index
__device__ __forceinline__ void next_best(const float* z, int n, float& v, int& i) {
  float bv = -INFINITY;
  int bi = n;
  for (int e = 0; e < n; ++e) {
    const float s = z[e];
    if ((s < v || (s == v && e > i)) && s > bv) bv = s, bi = e;
  }
  v = bv;
  i = min(bi, n - 1);
}

// kGroups, one wave: scores of one token's n <= 64 PER logits z (LDS, overwritten by the choice scores if PER > 1), the
// top k of them through put(j, output, score).  gm: LDS, groups floats.  Returns the weights of outputs from E on, added up.
template <int PER, typename F>
__device__ __forceinline__ float choose_groups(const ChooseArgs& c, float* z, float* gm, int E, int k, int lane, F&& put) {
  float s[PER], ch[PER], mx = -INFINITY, sum = 0.f;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int e = lane + 64 * i;
    s[i] = e < c.n ? z[e] : -INFINITY;
    mx = fmaxf(mx, s[i]);
  }
  mx = wave_max(mx);
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    s[i] = expf(s[i] - mx);
    sum += s[i];
  }
  const float inv = 1.f / wave_sum(sum);
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int e = lane + 64 * i;
    s[i] *= inv;
    ch[i] = e < c.n ? s[i] + (c.correction ? c.correction[e] : 0.f) : -INFINITY;
  }
  if (c.keep < c.groups) {
    // an output stays if fewer than `keep` groups come ahead of its own (ties: the lower group)
    const int size = c.n / c.groups;
    if constexpr (PER == 1) {
      const int mine = lane / size;
      float best = -INFINITY, own = -INFINITY;  // lane g: group g's best; and the own group's
      for (int g = 0; g < c.groups; ++g) {
        const float m = wave_max(mine == g ? ch[0] : -INFINITY);
        best = lane == g ? m : best;
        own = mine == g ? m : own;
      }
      int before = 0;
      for (int g = 0; g < c.groups; ++g) {
        const float m = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(best), g));
        before += m > own || (m == own && g < mine);
      }
      if (before >= c.keep) ch[0] = -INFINITY;
    } else {
      auto lds_fence = [] {
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "workgroup");
        __builtin_amdgcn_wave_barrier();
      };
#pragma unroll
      for (int i = 0; i < PER; ++i)
        if (lane + 64 * i < c.n) z[lane + 64 * i] = ch[i];
      lds_fence();
      for (int g = lane; g < c.groups; g += 64) {
        float m = -INFINITY;
        for (int e = 0; e < size; ++e) m = fmaxf(m, z[g * size + e]);
        gm[g] = m;
      }
      lds_fence();
#pragma unroll
      for (int i = 0; i < PER; ++i) {
        const int e = lane + 64 * i;
        if (e >= c.n) continue;
        const int g = e / size;
        const float own = gm[g];
        int before = 0;
        for (int o = 0; o < c.groups; ++o) before += gm[o] > own || (gm[o] == own && o < g);
        if (before >= c.keep) ch[i] = -INFINITY;
      }
    }
  }
  float own = 0.f;
  for (int j = 0; j < k; ++j) {
    float bv = ch[0];
#pragma unroll
    for (int i = 1; i < PER; ++i) bv = fmaxf(bv, ch[i]);
    bv = wave_max(bv);
    int be = j;  // (no number is the largest: any output)
#pragma unroll
    for (int i = PER - 1; i >= 0; --i) {
      const unsigned long long at = __ballot(ch[i] == bv && lane + 64 * i < c.n);
      if (at) be = 64 * i + __builtin_ctzll(at);
    }
#pragma unroll
    for (int i = 0; i < PER; ++i)
      if (be == lane + 64 * i) {
        put(j, be, s[i]);
        if (be >= E) own += s[i];
        ch[i] = -INFINITY;
      }
  }
  return wave_sum(own);
}

template <typename F>
__device__ __forceinline__ float choose_groups(const ChooseArgs& c, float* z, float* gm, int E, int k, int lane, F&& put) {
  return c.n <= 64 ? choose_groups<1>(c, z, gm, E, k, lane, put) : choose_groups<kSigMaxE / 64>(c, z, gm, E, k, lane, put);
}

// kGroups: logits lg [nt <= 16 tokens][n <= 16 NT outputs] on the matrix cores, rows of H (a multiple of 64) elements.
// The waves take 64 columns in turn; their partial sums meet in red (LDS).  Ends with a barrier behind its last write.
template <int NT, int LD>
__device__ __forceinline__ void router_tile(const uint16_t* x, int nt, const uint16_t* w, int n, int H, float (*lg)[LD],
                                            float (*red)[16][16 * NT + 1]) {
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const uint16_t* xr = x + (size_t)min(r, nt - 1) * H + g * 8;
  const uint16_t* wr[NT];
  f32x4 acc[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    wr[i] = w + (size_t)min(16 * i + r, n - 1) * H + g * 8;
    acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  constexpr int U = NT > 2 ? 1 : 4 / NT;  // loads of U x 64 columns in flight
#pragma unroll U
  for (int k = 64 * wv; k < H; k += 64 * kDispWaves) {
#pragma unroll
    for (int kk = 0; kk < 64; kk += 32) {
      const bf16x8 a = *reinterpret_cast<const bf16x8*>(xr + k + kk);
#pragma unroll
      for (int i = 0; i < NT; ++i) acc[i] = mfma16(a, *reinterpret_cast<const bf16x8*>(wr[i] + k + kk), acc[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) red[wv][4 * g + j][16 * i + r] = acc[i][j];
  __syncthreads();
  for (int u = threadIdx.x; u < nt * n; u += 64 * kDispWaves) {
    const int t = u / n, e = u % n;
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < kDispWaves; ++i) sum += red[i][t][e];
    lg[t][e] = sum;
  }
  __syncthreads();
}

// router logits of two token rows, any row length (a multiple of 8)
__device__ __forceinline__ void dot_rows2(const uint16_t* w, const uint16_t* x0, const uint16_t* x1, int H, int lane,
                                          float& s0, float& s1) {
  s0 = s1 = 0.f;
#pragma unroll 4
  for (int c = lane * 8; c < H; c += 512) {
    const u32x4 b = *reinterpret_cast<const u32x4*>(w + c), p = *reinterpret_cast<const u32x4*>(x0 + c),
                q = *reinterpret_cast<const u32x4*>(x1 + c);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      s0 += lo_bf(p[j]) * lo_bf(b[j]) + hi_bf(p[j]) * hi_bf(b[j]);
      s1 += lo_bf(q[j]) * lo_bf(b[j]) + hi_bf(q[j]) * hi_bf(b[j]);
    }
  }
  s0 = wave_sum(s0);
  s1 = wave_sum(s1);
}

template <int CH, int KIND = kSoftmax>  // 16-B chunks per lane per row: H = CH * 512 (0: any H)
__global__ void __launch_bounds__(64 * kDispWaves) moe_dispatch_small_kernel(
    float* __restrict__ topw, int* __restrict__ topi, uint16_t* __restrict__ xp, int* __restrict__ offsets,
    int* __restrict__ src, int* __restrict__ inv, const uint16_t* __restrict__ x,
    const uint16_t* __restrict__ wr, int T, int E, int k, int H, int e0, int n_local, MoePro pro, SigArgs sig = SigArgs{}, ChooseArgs cho = ChooseArgs{}) {
  constexpr bool SIG = KIND == kSigmoid;
  constexpr int ME = KIND != kSoftmax ? kSigMaxE : kMaxE, MK = KIND != kSoftmax ? kSigMaxTop : 8;
  __shared__ float lg[kSmallT][ME + SIG];
  __shared__ float s_gm[KIND == kGroups ? kDispWaves : 1][KIND == kGroups ? kSigMaxE : 1];
  __shared__ int s_topi[kSmallT * MK];
  __shared__ float s_topw[SIG ? kSmallT * MK : 1];
  __shared__ int cnt[ME + 1];
  __shared__ int base[ME + 1];
  __shared__ float red[16];
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
  if (pro.y != nullptr) {
    // 0. prologue: residual += y; x = rmsnorm(residual) * w (norm.hip's rounding), x -> pro.xn
    for (int t = 0; t < T; ++t) {
      u32x4 r[2];  // H <= 8192: at most two 8-element chunks per thread
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int c = (threadIdx.x + i * 64 * kDispWaves) * 8;
        if (c >= H) continue;
        const u32x4 a = *reinterpret_cast<const u32x4*>(pro.y + (size_t)t * H + c);
        const u32x4 b = *reinterpret_cast<const u32x4*>(pro.residual + (size_t)t * H + c);
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          r[i][q] = pack2(lo_bf(a[q]) + lo_bf(b[q]), hi_bf(a[q]) + hi_bf(b[q]));
          ss += lo_bf(r[i][q]) * lo_bf(r[i][q]) + hi_bf(r[i][q]) * hi_bf(r[i][q]);
        }
        *reinterpret_cast<u32x4*>(pro.residual + (size_t)t * H + c) = r[i];
      }
      const float rs = rsqrtf(block_sum(ss, red) / (float)H + pro.eps);
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int c = (threadIdx.x + i * 64 * kDispWaves) * 8;
        if (c >= H) continue;
        const u32x4 wv8 = *reinterpret_cast<const u32x4*>(pro.w + c);
        u32x4 o;
#pragma unroll
        for (int q = 0; q < 4; ++q)
          o[q] = pack2(bf2f(f2bf(lo_bf(r[i][q]) * rs)) * lo_bf(wv8[q]), bf2f(f2bf(hi_bf(r[i][q]) * rs)) * hi_bf(wv8[q]));
        *reinterpret_cast<u32x4*>(pro.xn + (size_t)t * H + c) = o;
      }
    }
    __syncthreads();  // x is read back below by other threads of this workgroup
    x = pro.xn;
  }
  // 1. router logits: lg[t][e] = bf16(x[t] . wr[e])
  for (int e = wv; e < (KIND == kGroups ? cho.n : SIG ? sig.rows : E); e += kDispWaves) {
    if constexpr (CH == 0) {
      for (int t = 0; t < T; t += 2) {
        float s0, s1;
        dot_rows2(wr + (size_t)e * H, x + (size_t)t * H, x + (size_t)min(t + 1, T - 1) * H, H, lane, s0, s1);
        if (lane == 0) lg[t][e] = s0;
        if (lane == 0 && t + 1 < T) lg[t + 1][e] = s1;
      }
      continue;
    }
    const uint16_t* we = wr + (size_t)e * H + lane * 8;
    constexpr int CN = CH > 0 ? CH : 1;
    u32x4 b[CN];
#pragma unroll
    for (int i = 0; i < CH; ++i) b[i] = *reinterpret_cast<const u32x4*>(we + i * 512);
    for (int t = 0; t < T; ++t) {
      const uint16_t* xt = x + (size_t)t * H + lane * 8;
      u32x4 a[CN];
#pragma unroll
      for (int i = 0; i < CH; ++i) a[i] = *reinterpret_cast<const u32x4*>(xt + i * 512);
      float acc = 0.f;
#pragma unroll
      for (int i = 0; i < CH; ++i)
#pragma unroll
        for (int q = 0; q < 4; ++q) acc += lo_bf(a[i][q]) * lo_bf(b[i][q]) + hi_bf(a[i][q]) * hi_bf(b[i][q]);
      acc = wave_sum(acc);
      if (lane == 0) lg[t][e] = KIND != kSoftmax ? acc : bf2f(f2bf(acc));
    }
  }
  for (int e = threadIdx.x; e <= n_local; e += blockDim.x) cnt[e] = 0;
  __syncthreads();
  // 2. softmax -> top-k -> renormalise (moe_route_kernel's math), one thread per token
  if constexpr (KIND == kGroups) {
    for (int t = wv; t < T; t += kDispWaves) {
      const float own = choose_groups(cho, lg[t], s_gm[wv], E, k, lane, [&](int j, int e, float s) {
        s_topi[t * k + j] = topi[t * k + j] = e;
        topw[t * k + j] = s;
      });
      if (cho.self_w && lane == 0) cho.self_w[t] = own;
    }
  } else if (SIG && threadIdx.x < T) {
    const int t = threadIdx.x;
    float v = INFINITY;
    int e = -1;
    for (int j = 0; j < k; ++j) {
      next_best(lg[t], E, v, e);
      s_topi[t * k + j] = topi[t * k + j] = e;
      s_topw[t * k + j] = topw[t * k + j] = sigmoid_of(v);
    }
    if (sig.gate) sig.gate[t] = sigmoid_of(lg[t][E]);
  } else if (threadIdx.x < T) {
    const int t = threadIdx.x;
    float mx = -INFINITY;
    for (int e = 0; e < E; ++e) mx = fmaxf(mx, lg[t][e]);
    float sum = 0.f;
    for (int e = 0; e < E; ++e) sum += __expf(lg[t][e] - mx);
    const float rinv = 1.f / sum;
    float picked = 0.f, wsel[8];
    int isel[8];
    unsigned long long used = 0ull;
    for (int j = 0; j < k; ++j) {
      int best = 0;
      float bv = -1.f;
      for (int e = 0; e < E; ++e) {
        const float v = __expf(lg[t][e] - mx);
        if (!((used >> e) & 1ull) && v > bv) { bv = v; best = e; }
      }
      used |= 1ull << best;
      isel[j] = best;
      wsel[j] = bv * rinv;
      picked += bv * rinv;
    }
    const float rn = picked > 0.f ? 1.f / picked : 0.f;
    for (int j = 0; j < k; ++j) {
      topi[t * k + j] = isel[j];
      topw[t * k + j] = wsel[j] * rn;
      s_topi[t * k + j] = isel[j];
    }
  }
  __syncthreads();
  // 3. counting sort of the T*k slots by local expert (moe_sort_kernel), slot order kept
  const int n_slots = T * k;
  if constexpr (KIND == kGroups) {  // any order inside an expert: no value depends on it
    constexpr int PER = kSmallT * kSigMaxTop / (64 * kDispWaves);
    int rank[PER];
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int s = threadIdx.x + 64 * kDispWaves * i, e = s < n_slots ? s_topi[s] : E;
      rank[i] = e < E ? atomicAdd(&cnt[e], 1) : -1;
    }
    __syncthreads();
    if (threadIdx.x == 0) {
      int acc = 0;
      for (int e = 0; e < E; ++e) {
        base[e] = acc;
        offsets[e] = acc;
        acc += cnt[e];
      }
      offsets[E] = acc;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int s = threadIdx.x + 64 * kDispWaves * i;
      if (s >= n_slots) continue;
      const int row = rank[i] < 0 ? -1 : base[s_topi[s]] + rank[i];
      inv[s] = row;
      if (row >= 0) src[row] = s;
      s_topi[s] = row;
    }
  } else if (threadIdx.x == 0) {
    for (int s = 0; s < n_slots; ++s) {
      const int e = s_topi[s] - e0;
      if (e >= 0 && e < n_local) ++cnt[e];
    }
    int acc = 0;
    for (int e = 0; e < n_local; ++e) {
      base[e] = acc;
      offsets[e] = acc;
      acc += cnt[e];
      cnt[e] = 0;
    }
    offsets[n_local] = acc;
    for (int s = 0; s < n_slots; ++s) {
      const int e = s_topi[s] - e0;
      if (e >= 0 && e < n_local) {
        const int row = base[e] + cnt[e]++;
        inv[s] = row;
        src[row] = s;
        s_topi[s] = row;  // reused: slot -> row for the gather below
      } else {
        inv[s] = -1;
        s_topi[s] = -1;
      }
    }
  }
  __syncthreads();
  // 4. gather: xp[row(s)] = x[s / k]
  const int vpr = H / 8;
  for (int i = threadIdx.x; i < n_slots * vpr; i += blockDim.x) {
    const int s = i / vpr, c = (i % vpr) * 8;
    const int row = s_topi[s];
    if (row < 0) continue;
    u32x4 v = *reinterpret_cast<const u32x4*>(x + (size_t)(s / k) * H + c);
    if constexpr (SIG) {
#pragma unroll
      for (int q = 0; q < 4; ++q) v[q] = pack2(s_topw[s] * lo_bf(v[q]), s_topw[s] * hi_bf(v[q]));
    }
    *reinterpret_cast<u32x4*>(xp + (size_t)row * H + c) = v;
  }
}

bool moe_dispatch_small_takes(int T, int E, int k, int H) {
  return T >= 1 && T <= kSmallT && E <= kMaxE && k <= 8 && (H == 1024 || H == 2048 || H == 4096 || H == 8192);
}

void launch_moe_dispatch_small(float* topw, int* topi, void* xp, int* offsets, int* src, int* inv, const void* x,
                               const void* wr, int T, int E, int k, int H, int e0, int n_local, const void* pro_y,
                               void* pro_res, const void* pro_w, float pro_eps, void* pro_xn, hipStream_t st) {
  const MoePro pro{(const uint16_t*)pro_y, (uint16_t*)pro_res, (const uint16_t*)pro_w, pro_eps, (uint16_t*)pro_xn};
#define MLOP_DISP(CH)                                                                                       \
  moe_dispatch_small_kernel<CH><<<1, 64 * kDispWaves, 0, st>>>(topw, topi, (uint16_t*)xp, offsets, src, inv, \
                                                               (const uint16_t*)x, (const uint16_t*)wr, T, E, k, \
                                                               H, e0, n_local, pro)
  switch (H) {
    case 1024: MLOP_DISP(2); break;
    case 2048: MLOP_DISP(4); break;
    case 4096: MLOP_DISP(8); break;
    default: MLOP_DISP(16); break;
  }
#undef MLOP_DISP
}

void launch_moe_dispatch_small_sigmoid(float* topw, int* topi, void* xp, int* offsets, int* src, int* inv, float* gate,
                                       const void* x, const void* wr, int T, int E, int rows, int k, int H,
                                       hipStream_t st) {
  const SigArgs sig{gate, nullptr, rows};
#define MLOP_DISP(CH)                                                                                             \
  moe_dispatch_small_kernel<CH, kSigmoid><<<1, 64 * kDispWaves, 0, st>>>(topw, topi, (uint16_t*)xp, offsets, src, inv, \
                                                                     (const uint16_t*)x, (const uint16_t*)wr, T, E, k, \
                                                                     H, 0, E, MoePro{}, sig)
  switch (H) {
    case 1024: MLOP_DISP(2); break;
    case 2048: MLOP_DISP(4); break;
    case 4096: MLOP_DISP(8); break;
    case 8192: MLOP_DISP(16); break;
    default: MLOP_DISP(0); break;
  }
#undef MLOP_DISP
}

// ---------------------------------------------------------------------------
// MoE dispatch for 16 < T <= kMidT tokens (decode batches and prefill chunks) in ONE launch.  At batch 64 the separate
// route is five ~5 us graph nodes per layer (router GEMM + its split-K reduce, top-k, sort,
// gather: profiles/r05_windows.md), each a few us of work at most.  Here:
//   workgroup w (tokens kMidTok w .., moe_mid_tok): the optional add + RMSNorm prologue, router logits
//     (wave e = expert e: the router row loaded once, bf16-rounded as the separate projection
//     stores them), softmax / top-k / renormalise -> topw, topi (written through, sc1);
//   the LAST workgroup (one agent-scope ticket per launch, reset by it: graph-safe; dispatch
//     order and co-residency are not assumed) counts the T*k slots per local expert and writes
//     offsets, inv (slot -> permuted row) and arow (permuted row -> token row).
// There is no gathered copy: the grouped gate_up GEMM reads x rows through arow.  Rows inside
// an expert come in ticket order (LDS atomics), which changes no value: each row's product is
// independent of its position and the combine gathers by inv.
constexpr int kMidT = 16384;
static int g_mid_max_t = kMidT;  // moe_mid_max_tokens op: in-process A/B of the range
// moe_mid_tok op: tokens per workgroup (2, 4 or 8; the router row is loaded once per
// workgroup, token rows two at a time).  Fewer workgroups = fewer router-row reloads and
// fewer agent-scope tickets on the one counter, more sequential prologue tokens per workgroup.
// 0 (default) = by T: 8 from 2,048 tokens, 4 from 512, else 2.  Mixtral batch 1024 windows,
// 2 / 4 / 8: the 3,060-token mixed step 42.3 / 32.3 / 29.3 us, the 1,024-token decode step
// 17.6 / 13.7 / 14.7 us (profiles/r06_moe_spill.md)
static int g_mid_tok = 0;
int moe_mid_tok(int set) {
  if (set == 0 || set == 2 || set == 4 || set == 8) g_mid_tok = set;
  return g_mid_tok;
}
int moe_mid_max_tokens(int set) {
  if (set >= 0) g_mid_max_t = set < kMidT ? set : kMidT;
  return g_mid_max_t;
}

template <int CH, int kMidTok, int KIND = kSoftmax>  // CH 0: any H; < 0: router_tile of 16 * -CH outputs (kGroups)
__global__ void __launch_bounds__(64 * kDispWaves, CH < 0 ? 4 : 1) moe_dispatch_mid_kernel(
    float* __restrict__ topw, int* __restrict__ topi, int* __restrict__ offsets, int* __restrict__ arow,
    int* __restrict__ inv, const uint16_t* __restrict__ x, const uint16_t* __restrict__ wr, int T, int E, int k,
    int H, int e0, int n_local, MoePro pro, int* __restrict__ ticket, SigArgs sig = SigArgs{}, ChooseArgs cho = ChooseArgs{}) {
  constexpr bool SIG = KIND == kSigmoid;
  constexpr int ME = KIND != kSoftmax ? kSigMaxE : kMaxE;
  __shared__ float lg[kMidTok][ME + SIG];
  __shared__ float s_gm[KIND == kGroups ? kDispWaves : 1][KIND == kGroups ? kSigMaxE : 1];
  __shared__ int cnt[ME + 1];
  __shared__ int base[ME + 1];
  __shared__ float red[16];
  __shared__ int last;
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
  const int t0 = blockIdx.x * kMidTok, nt = min(kMidTok, T - t0);
  if (pro.y != nullptr) {
    // prologue for this workgroup's tokens: residual += y; x = rmsnorm(residual) * w
    for (int t = t0; t < t0 + nt; ++t) {
      u32x4 r[2];
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int c = (threadIdx.x + i * 64 * kDispWaves) * 8;
        if (c >= H) continue;
        const u32x4 a = *reinterpret_cast<const u32x4*>(pro.y + (size_t)t * H + c);
        const u32x4 b = *reinterpret_cast<const u32x4*>(pro.residual + (size_t)t * H + c);
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          r[i][q] = pack2(lo_bf(a[q]) + lo_bf(b[q]), hi_bf(a[q]) + hi_bf(b[q]));
          ss += lo_bf(r[i][q]) * lo_bf(r[i][q]) + hi_bf(r[i][q]) * hi_bf(r[i][q]);
        }
        *reinterpret_cast<u32x4*>(pro.residual + (size_t)t * H + c) = r[i];
      }
      const float rs = rsqrtf(block_sum(ss, red) / (float)H + pro.eps);
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int c = (threadIdx.x + i * 64 * kDispWaves) * 8;
        if (c >= H) continue;
        const u32x4 wv8 = *reinterpret_cast<const u32x4*>(pro.w + c);
        u32x4 o;
#pragma unroll
        for (int q = 0; q < 4; ++q)
          o[q] = pack2(bf2f(f2bf(lo_bf(r[i][q]) * rs)) * lo_bf(wv8[q]), bf2f(f2bf(hi_bf(r[i][q]) * rs)) * hi_bf(wv8[q]));
        *reinterpret_cast<u32x4*>(pro.xn + (size_t)t * H + c) = o;
      }
    }
    __syncthreads();  // this workgroup's x rows are read back below by other threads
    x = pro.xn;
  }
  // router logits of this workgroup's tokens
  // rows past a whole round of the waves (a gate behind 8 experts, say) are dealt to them by token pairs
  const int n_rows = KIND == kGroups ? cho.n : SIG ? sig.rows : E;
  const int n_rounds = CH < 0 ? 0 : KIND != kSoftmax ? n_rows / kDispWaves * kDispWaves : E;
  if constexpr (CH < 0) {
    __shared__ float part[kDispWaves][16][16 * -CH + 1];
    router_tile<-CH>(x + (size_t)t0 * H, nt, wr, cho.n, H, lg, part);
  } else if constexpr (KIND != kSoftmax) {
    const int pairs = (nt + 1) >> 1;
    for (int u = wv; u < (n_rows - n_rounds) * pairs; u += kDispWaves) {
      const int e = n_rounds + u / pairs, tp = u % pairs * 2;
      float s0, s1;
      dot_rows2(wr + (size_t)e * H, x + (size_t)(t0 + tp) * H, x + (size_t)(t0 + min(tp + 1, nt - 1)) * H, H, lane, s0, s1);
      if (lane == 0) lg[tp][e] = s0;
      if (lane == 0 && tp + 1 < nt) lg[tp + 1][e] = s1;
    }
  }
  for (int e = wv; e < n_rounds; e += kDispWaves) {
    if constexpr (CH == 0) {
      for (int tp = 0; tp < nt; tp += 2) {
        float s0, s1;
        dot_rows2(wr + (size_t)e * H, x + (size_t)(t0 + tp) * H, x + (size_t)(t0 + min(tp + 1, nt - 1)) * H, H, lane, s0, s1);
        if (lane == 0) lg[tp][e] = s0;
        if (lane == 0 && tp + 1 < nt) lg[tp + 1][e] = s1;
      }
      continue;
    }
    const uint16_t* we = wr + (size_t)e * H + lane * 8;
    constexpr int CN = CH > 0 ? CH : 1;
    u32x4 b[CN];
#pragma unroll
    for (int i = 0; i < CH; ++i) b[i] = *reinterpret_cast<const u32x4*>(we + i * 512);
    // token rows two at a time, both rows' chunks in flight together (with the router row's
    // on the first pair: one latency, not three)
#pragma unroll 1
    for (int tp = 0; tp < kMidTok; tp += 2) {
      u32x4 a[2][CN];
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int i = 0; i < CH; ++i)
          a[t][i] = *reinterpret_cast<const u32x4*>(x + (size_t)(t0 + min(tp + t, nt - 1)) * H + lane * 8 + i * 512);
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        float acc = 0.f;
#pragma unroll
        for (int i = 0; i < CH; ++i)
#pragma unroll
          for (int q = 0; q < 4; ++q)
            acc += lo_bf(a[t][i][q]) * lo_bf(b[i][q]) + hi_bf(a[t][i][q]) * hi_bf(b[i][q]);
        acc = wave_sum(acc);
        if (lane == 0 && tp + t < nt) lg[tp + t][e] = KIND != kSoftmax ? acc : bf2f(f2bf(acc));
      }
    }
  }
  __syncthreads();
  const auto rs_topi = __builtin_amdgcn_make_buffer_rsrc((void*)topi, 0, T * k * 4, 0x00020000);
  const auto rs_topw = __builtin_amdgcn_make_buffer_rsrc((void*)topw, 0, T * k * 4, 0x00020000);
  if constexpr (KIND == kGroups) {
    for (int t = wv; t < nt; t += kDispWaves) {
      const float own = choose_groups(cho, lg[t], s_gm[wv], E, k, lane, [&](int j, int e, float s) {
        const uint32_t at = (uint32_t)(((t0 + t) * k + j) * 4);
        topw[(t0 + t) * k + j] = s;
        __builtin_amdgcn_raw_buffer_store_b32(e, rs_topi, at, 0, 16 /* sc1 */);
      });
      if (cho.self_w && lane == 0) cho.self_w[t0 + t] = own;
    }
  } else if (SIG && threadIdx.x < nt) {
    const int t = threadIdx.x;
    float v = INFINITY;
    int e = -1;
    for (int j = 0; j < k; ++j) {
      next_best(lg[t], E, v, e);
      const uint32_t at = (uint32_t)(((t0 + t) * k + j) * 4);
      __builtin_amdgcn_raw_buffer_store_b32(__float_as_uint(sigmoid_of(v)), rs_topw, at, 0, 16 /* sc1 */);
      __builtin_amdgcn_raw_buffer_store_b32(e, rs_topi, at, 0, 16 /* sc1 */);
    }
    if (sig.gate) sig.gate[t0 + t] = sigmoid_of(lg[t][E]);
  } else if (threadIdx.x < nt) {  // moe_route_kernel's math
    const int t = threadIdx.x;
    float mx = -INFINITY;
    for (int e = 0; e < E; ++e) mx = fmaxf(mx, lg[t][e]);
    float sum = 0.f;
    for (int e = 0; e < E; ++e) sum += __expf(lg[t][e] - mx);
    const float rinv = 1.f / sum;
    float picked = 0.f, wsel[8];
    int isel[8];
    unsigned long long used = 0ull;
    for (int j = 0; j < k; ++j) {
      int best = 0;
      float bv = -1.f;
      for (int e = 0; e < E; ++e) {
        const float v = __expf(lg[t][e] - mx);
        if (!((used >> e) & 1ull) && v > bv) { bv = v; best = e; }
      }
      used |= 1ull << best;
      isel[j] = best;
      wsel[j] = bv * rinv;
      picked += bv * rinv;
    }
    const float rn = picked > 0.f ? 1.f / picked : 0.f;
    for (int j = 0; j < k; ++j) {
      topw[(t0 + t) * k + j] = wsel[j] * rn;
      // written through (sc1) for the sorting workgroup, which may sit on another XCD
      __builtin_amdgcn_raw_buffer_store_b32(isel[j], rs_topi, (uint32_t)(((t0 + t) * k + j) * 4), 0, 16 /* sc1 */);
    }
  }
  // every wave drains its stores, then one lane takes the ticket (the K-half hand-off of
  // gemm_w4.hip: sc1 stores, vmcnt(0), barrier, relaxed agent-scope counter, sc1 loads)
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  if (threadIdx.x == 0) {
    const int tk = __hip_atomic_fetch_add(ticket, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    last = tk == (int)gridDim.x - 1;
    if (last) __hip_atomic_store(ticket, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);  // next launch
  }
  __syncthreads();
  if (!last) return;
  // counting sort of the T*k slots by local expert
  const int n_slots = T * k;
  // kGroups: counters in kRep copies, a lane's by its number (few experts: lanes of a wave rarely meet)
  constexpr int kRep = CH < 0 ? 8 : 1;
  __shared__ int rep_cnt[kRep > 1 ? kRep * 64 : 1], rep_base[kRep > 1 ? kRep * 64 : 1];
  const int rep = threadIdx.x % kRep;
  for (int e = threadIdx.x; e <= n_local; e += blockDim.x) cnt[e] = 0;
  if (kRep > 1)
    for (int e = threadIdx.x; e < kRep * 64; e += blockDim.x) rep_cnt[e] = 0;
  __syncthreads();
  // the sc1 loads in batches of kSortChunk per thread, all in flight before the first use: one
  // at a time, each load's latency was paid per slot (a 3,060-token mixed step: 12 slots per
  // thread and pass, ~40 of the launch's 52 us)
  constexpr int kSortChunk = CH < 0 ? 24 : 8;
  auto load_chunk = [&](int s0, int (&ev)[kSortChunk]) {
#pragma unroll
    for (int j = 0; j < kSortChunk; ++j) {
      const int s = s0 + j * (int)blockDim.x + (int)threadIdx.x;  // past n_slots: out of range, reads 0
      ev[j] = __builtin_amdgcn_raw_buffer_load_b32(rs_topi, (uint32_t)(s * 4), 0, 16 /* sc1 */) - e0;
    }
  };
  for (int s0 = 0; s0 < n_slots; s0 += kSortChunk * (int)blockDim.x) {
    int ev[kSortChunk];
    load_chunk(s0, ev);
#pragma unroll
    for (int j = 0; j < kSortChunk; ++j) {
      const int s = s0 + j * (int)blockDim.x + (int)threadIdx.x, e = ev[j];
      // rank in its expert (in its copy's part of it)
      if (s < n_slots) inv[s] = (e >= 0 && e < n_local) ? atomicAdd(kRep > 1 ? &rep_cnt[e * kRep + rep] : &cnt[e], 1) : -1;
    }
  }
  __syncthreads();
  if constexpr (kRep > 1) {
    if (threadIdx.x < 64) {  // lane = expert
      int n = 0, before;
      if (lane < n_local)
#pragma unroll
        for (int r = 0; r < kRep; ++r) n += rep_cnt[lane * kRep + r];
      before = n;
      for (int o = 1; o < 64; o <<= 1) {
        const int v = __shfl_up(before, o);
        if (lane >= o) before += v;
      }
      const int total = __shfl(before, 63);
      before -= n;
      if (lane < n_local) {
        offsets[lane] = before;
#pragma unroll
        for (int r = 0; r < kRep; ++r) {
          rep_base[lane * kRep + r] = before;
          before += rep_cnt[lane * kRep + r];
        }
      }
      if (lane == 0) offsets[n_local] = total;
    }
  } else if (threadIdx.x == 0) {
    int acc = 0;
    for (int e = 0; e < n_local; ++e) {
      base[e] = acc;
      offsets[e] = acc;
      acc += cnt[e];
    }
    offsets[n_local] = acc;
  }
  __syncthreads();
  for (int s0 = 0; s0 < n_slots; s0 += kSortChunk * (int)blockDim.x) {
    int ev[kSortChunk], rk[kSortChunk];
    load_chunk(s0, ev);
#pragma unroll
    for (int j = 0; j < kSortChunk; ++j) {  // this thread's own pass-1 stores: plain loads see them
      const int s = s0 + j * (int)blockDim.x + (int)threadIdx.x;
      rk[j] = s < n_slots ? inv[s] : -1;
    }
    float wt[kSortChunk];
    if constexpr (SIG) {
#pragma unroll
      for (int j = 0; j < kSortChunk; ++j)
        wt[j] = __uint_as_float(__builtin_amdgcn_raw_buffer_load_b32(
            rs_topw, (uint32_t)((s0 + j * (int)blockDim.x + (int)threadIdx.x) * 4), 0, 16 /* sc1 */));
    }
#pragma unroll
    for (int j = 0; j < kSortChunk; ++j) {
      const int s = s0 + j * (int)blockDim.x + (int)threadIdx.x, e = ev[j];
      if (s < n_slots && e >= 0 && e < n_local) {
        const int row = (kRep > 1 ? rep_base[e * kRep + rep] : base[e]) + rk[j];
        inv[s] = row;
        arow[row] = s / k;
        if constexpr (SIG) sig.row_w[row] = wt[j];
      }
    }
  }
}

bool moe_dispatch_mid_takes(int T, int E, int k, int H) {
  return T > kSmallT && T <= g_mid_max_t && E <= kMaxE && k <= 8 && (H == 1024 || H == 2048 || H == 4096 || H == 8192);
}

void launch_moe_dispatch_mid(float* topw, int* topi, int* offsets, int* arow, int* inv, const void* x, const void* wr,
                             int T, int E, int k, int H, int e0, int n_local, const void* pro_y, void* pro_res,
                             const void* pro_w, float pro_eps, void* pro_xn, hipStream_t st) {
  float* ws = nullptr;
  int* ticket = nullptr;
  int cus = 0;
  if (!gemm_sk_scratch(&ws, &ticket, &cus)) throw std::runtime_error("moe_dispatch_mid: stream-K scratch not reserved");
  const MoePro pro{(const uint16_t*)pro_y, (uint16_t*)pro_res, (const uint16_t*)pro_w, pro_eps, (uint16_t*)pro_xn};
  const int tok = g_mid_tok ? g_mid_tok : T >= 2048 ? 8 : T >= 512 ? 4 : 2, grid = (T + tok - 1) / tok;
#define MLOP_DISP_T(CH, TOK)                                                                                         \
  moe_dispatch_mid_kernel<CH, TOK><<<grid, 64 * kDispWaves, 0, st>>>(topw, topi, offsets, arow, inv, (const uint16_t*)x, \
                                                                     (const uint16_t*)wr, T, E, k, H, e0, n_local, pro, ticket)
#define MLOP_DISP(CH)                       \
  if (tok == 8) MLOP_DISP_T(CH, 8);         \
  else if (tok == 4) MLOP_DISP_T(CH, 4);    \
  else MLOP_DISP_T(CH, 2);
  switch (H) {
    case 1024: MLOP_DISP(2); break;
    case 2048: MLOP_DISP(4); break;
    case 4096: MLOP_DISP(8); break;
    default: MLOP_DISP(16); break;
  }
#undef MLOP_DISP
#undef MLOP_DISP_T
}

void launch_moe_dispatch_mid_sigmoid(float* topw, int* topi, int* offsets, int* arow, float* row_w, int* inv, float* gate,
                                     const void* x, const void* wr, int T, int E, int rows, int k, int H, hipStream_t st) {
  float* ws = nullptr;
  int* ticket = nullptr;
  int cus = 0;
  if (!gemm_sk_scratch(&ws, &ticket, &cus)) throw std::runtime_error("moe_dispatch_mid: stream-K scratch not reserved");
  const SigArgs sig{gate, row_w, rows};
  const int tok = T >= 2048 ? 8 : T >= 512 ? 4 : 2, grid = (T + tok - 1) / tok;
#define MLOP_DISP_T(CH, TOK)                                                                                           \
  moe_dispatch_mid_kernel<CH, TOK, kSigmoid><<<grid, 64 * kDispWaves, 0, st>>>(topw, topi, offsets, arow, inv,               \
                                                                           (const uint16_t*)x, (const uint16_t*)wr, T, E, \
                                                                           k, H, 0, E, MoePro{}, ticket, sig)
#define MLOP_DISP(CH)                       \
  if (tok == 8) MLOP_DISP_T(CH, 8);         \
  else if (tok == 4) MLOP_DISP_T(CH, 4);    \
  else MLOP_DISP_T(CH, 2);
  switch (H) {
    case 1024: MLOP_DISP(2); break;
    case 2048: MLOP_DISP(4); break;
    case 4096: MLOP_DISP(8); break;
    case 8192: MLOP_DISP(16); break;
    default: MLOP_DISP(0); break;
  }
#undef MLOP_DISP
#undef MLOP_DISP_T
}

void launch_moe_dispatch_small_groups(float* topw, int* topi, void* xp, int* offsets, int* src, int* inv, const void* x,
                                      const void* wr, int T, int E, int k, int H, const ChooseArgs& cho, hipStream_t st) {
#define MLOP_DISP(CH)                                                                                               \
  moe_dispatch_small_kernel<CH, kGroups><<<1, 64 * kDispWaves, 0, st>>>(topw, topi, (uint16_t*)xp, offsets, src, inv, \
                                                                        (const uint16_t*)x, (const uint16_t*)wr, T, E, k, \
                                                                        H, 0, E, MoePro{}, SigArgs{}, cho)
  switch (H) {
    case 1024: MLOP_DISP(2); break;
    case 2048: MLOP_DISP(4); break;
    case 4096: MLOP_DISP(8); break;
    case 8192: MLOP_DISP(16); break;
    default: MLOP_DISP(0); break;
  }
#undef MLOP_DISP
}

void launch_moe_dispatch_mid_groups(float* topw, int* topi, int* offsets, int* arow, int* inv, const void* x, const void* wr,
                                    int T, int E, int k, int H, const ChooseArgs& cho, hipStream_t st) {
  float* ws = nullptr;
  int* ticket = nullptr;
  int cus = 0;
  if (!gemm_sk_scratch(&ws, &ticket, &cus)) throw std::runtime_error("moe_dispatch_mid: stream-K scratch not reserved");
#define MLOP_DISP(CH, TOK)                                                                                                \
  moe_dispatch_mid_kernel<CH, TOK, kGroups><<<(T + TOK - 1) / TOK, 64 * kDispWaves, 0, st>>>(                               \
      topw, topi, offsets, arow, inv, (const uint16_t*)x, (const uint16_t*)wr, T, E, k, H, 0, E, MoePro{}, ticket, SigArgs{}, \
      cho)
  if (T > 1024 && H % 64 == 0 && cho.n <= 64) {  // tiles of 16 tokens
    if (cho.n <= 16) MLOP_DISP(-1, 16);
    else if (cho.n <= 32) MLOP_DISP(-2, 16);
    else MLOP_DISP(-4, 16);
  } else {
#define MLOP_DISP_T(CH) \
  if (T > 1024) MLOP_DISP(CH, 8); else MLOP_DISP(CH, 2)
    switch (H) {
      case 1024: MLOP_DISP_T(2); break;
      case 2048: MLOP_DISP_T(4); break;
      case 4096: MLOP_DISP_T(8); break;
      case 8192: MLOP_DISP_T(16); break;
      default: MLOP_DISP_T(0); break;
    }
#undef MLOP_DISP_T
  }
#undef MLOP_DISP
}

// fp32 forms of the sigmoid and the grouped routing: one thread (wave) per token over its logits, the counting sort, a
// gather that may weight the rows, and the experts' products on fp32 FMAs
__global__ void __launch_bounds__(256) moe_route_groups_kernel(float* __restrict__ topw, int* __restrict__ topi,
                                                              const float* __restrict__ logits, int T, int E, int k,
                                                              ChooseArgs cho) {
  __shared__ float z[4][kSigMaxE], gm[4][kSigMaxE];
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, t = blockIdx.x * 4 + wv;
  if (t >= T) return;  // whole waves; no barrier below
  for (int e = lane; e < cho.n; e += 64) z[wv][e] = logits[(size_t)t * cho.n + e];
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "workgroup");
  __builtin_amdgcn_wave_barrier();
  const float own = choose_groups(cho, z[wv], gm[wv], E, k, lane, [&](int j, int e, float s) {
    topi[t * k + j] = e;
    topw[t * k + j] = s;
  });
  if (cho.self_w && lane == 0) cho.self_w[t] = own;
}

void launch_moe_route_groups(float* topw, int* topi, const float* logits, int T, int E, int k, const ChooseArgs& cho,
                             hipStream_t st) {
  if (T == 0) return;
  moe_route_groups_kernel<<<(T + 3) / 4, 256, 0, st>>>(topw, topi, logits, T, E, k, cho);
}

__global__ void __launch_bounds__(128) moe_route_sigmoid_kernel(float* __restrict__ topw, int* __restrict__ topi,
                                                               float* __restrict__ gate, const float* __restrict__ logits,
                                                               int T, int E, int rows, int k) {
  const int t = blockIdx.x * blockDim.x + threadIdx.x;
  if (t >= T) return;
  const float* l = logits + (size_t)t * rows;
  float v = INFINITY;
  int e = -1;
  for (int j = 0; j < k; ++j) {
    next_best(l, E, v, e);
    topi[t * k + j] = e;
    topw[t * k + j] = 1.f / (1.f + expf(-v));
  }
  if (gate) gate[t] = 1.f / (1.f + expf(-l[E]));
}

void launch_moe_route_sigmoid(float* topw, int* topi, float* gate, const float* logits, int T, int E, int rows, int k,
                              hipStream_t st) {
  if (T == 0) return;
  moe_route_sigmoid_kernel<<<(T + 127) / 128, 128, 0, st>>>(topw, topi, gate, logits, T, E, rows, k);
}

__global__ void __launch_bounds__(256) moe_gather_scaled_kernel(float* __restrict__ xp, const float* __restrict__ x,
                                                               const int* __restrict__ src, const float* __restrict__ topw,
                                                               const int* __restrict__ offsets, int n_local, int k, int H) {
  const int r = blockIdx.x;
  if (r >= offsets[n_local]) return;
  const int s = src[r];
  const float w = topw ? topw[s] : 1.f;
  for (int c = threadIdx.x; c < H; c += blockDim.x) xp[(size_t)r * H + c] = w * x[(size_t)(s / k) * H + c];
}

void launch_moe_permute_scaled(float* xp, int* offsets, int* src, int* inv, const float* x, const int* topi,
                               const float* topw, int T, int k, int H, int E, hipStream_t st) {
  moe_sort_kernel<<<1, 1024, 0, st>>>(offsets, src, inv, topi, T * k, 0, E);
  if (T * k > 0) moe_gather_scaled_kernel<<<T * k, 256, 0, st>>>(xp, x, src, topw, offsets, E, k, H);
}

// a 32 x 64 tile of one expert's rows (blockIdx.y: the tile among all experts'), 8 outputs per thread
__global__ void __launch_bounds__(256) grouped_plain_kernel(float* __restrict__ out, const float* __restrict__ a,
                                                           const float* __restrict__ w, const int* __restrict__ offsets,
                                                           int G, int N, int K) {
  __shared__ float sa[32][33], sb[64][33];
  int t = blockIdx.y, e = 0;
  for (; e < G; ++e) {
    const int tiles = (offsets[e + 1] - offsets[e] + 31) / 32;
    if (t < tiles) break;
    t -= tiles;
  }
  if (e >= G) return;
  const int m0 = offsets[e] + 32 * t, m_end = offsets[e + 1], n0 = blockIdx.x * 64, tid = threadIdx.x;
  const int tm = tid >> 5, tn = tid & 31;  // rows tm + 8 i, columns tn + 32 j
  const float* we = w + (size_t)e * N * K;
  float acc[4][2] = {};
  for (int k0 = 0; k0 < K; k0 += 32) {
    __syncthreads();
    for (int i = tid; i < 32 * 32; i += 256) {
      const int r = i >> 5, c = i & 31;
      sa[r][c] = m0 + r < m_end && k0 + c < K ? a[(size_t)(m0 + r) * K + k0 + c] : 0.f;
    }
    for (int i = tid; i < 64 * 32; i += 256) {
      const int r = i >> 5, c = i & 31;
      sb[r][c] = n0 + r < N && k0 + c < K ? we[(size_t)(n0 + r) * K + k0 + c] : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int c = 0; c < 32; ++c)
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = fmaf(sa[tm + 8 * i][c], sb[tn + 32 * j][c], acc[i][j]);
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
      if (m0 + tm + 8 * i < m_end && n0 + tn + 32 * j < N) out[(size_t)(m0 + tm + 8 * i) * N + n0 + tn + 32 * j] = acc[i][j];
}

void launch_grouped_plain(float* out, const float* a, const float* w, const int* offsets, int G, int R, int N, int K,
                          hipStream_t st) {
  if (R == 0) return;
  grouped_plain_kernel<<<dim3(cdiv(N, 64), cdiv(R, 32) + G), 256, 0, st>>>(out, a, w, offsets, G, N, K);
}

// combine fused with the decoder's residual add + RMSNorm (one workgroup per token row, 8
// elements per thread: at decode sizes every row's reads are in flight at once):
//   m = bf16(sum_j topw[t, j] * y[inv[t*k + j]])   (moe_combine_kernel's rounding)
//   residual[t] = bf16(residual[t] + m);  out[t] = bf16(bf16(residual[t] * rsqrt(mean sq + eps)) * w)
// SLABS: y is not formed; the grouped down GEMM's fp32 split-K slabs ws[s][R][H] are summed
// here (splitk_reduce_kernel's rounding: one bf16 rounding of the sum), one launch fewer
template <bool SLABS>
__global__ void __launch_bounds__(1024) moe_combine_add_rmsnorm_kernel(
    uint16_t* __restrict__ out, uint16_t* __restrict__ residual, const uint16_t* __restrict__ y,
    const int* __restrict__ inv, const float* __restrict__ topw, const uint16_t* __restrict__ w, float eps,
    int k, int H, const float* __restrict__ ws, int splits, int R) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, c = threadIdx.x * 8;
  float acc[8] = {0, 0, 0, 0, 0, 0, 0, 0};
  for (int j = 0; j < k; ++j) {
    const int row = inv[t * k + j];
    if (row < 0) continue;
    const float wt = topw[t * k + j];
    u32x4 v;
    if constexpr (SLABS) {
      float a[8] = {0, 0, 0, 0, 0, 0, 0, 0};
      for (int sp = 0; sp < splits; ++sp) {
        const float4* p = reinterpret_cast<const float4*>(ws + ((size_t)sp * R + row) * H + c);
        const float4 x0 = p[0], x1 = p[1];
        a[0] += x0.x; a[1] += x0.y; a[2] += x0.z; a[3] += x0.w;
        a[4] += x1.x; a[5] += x1.y; a[6] += x1.z; a[7] += x1.w;
      }
#pragma unroll
      for (int q = 0; q < 4; ++q) v[q] = pack2(a[2 * q], a[2 * q + 1]);
    } else {
      v = *reinterpret_cast<const u32x4*>(y + (size_t)row * H + c);
    }
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      acc[2 * q] += wt * lo_bf(v[q]);
      acc[2 * q + 1] += wt * hi_bf(v[q]);
    }
  }
  const u32x4 res = *reinterpret_cast<const u32x4*>(residual + (size_t)t * H + c);
  const u32x4 wv = *reinterpret_cast<const u32x4*>(w + c);
  u32x4 r;
  float ss = 0.f;
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const uint32_t m = pack2(acc[2 * q], acc[2 * q + 1]);
    r[q] = pack2(lo_bf(m) + lo_bf(res[q]), hi_bf(m) + hi_bf(res[q]));
    ss += lo_bf(r[q]) * lo_bf(r[q]) + hi_bf(r[q]) * hi_bf(r[q]);
  }
  *reinterpret_cast<u32x4*>(residual + (size_t)t * H + c) = r;
  const float rs = rsqrtf(block_sum(ss, scratch) / (float)H + eps);
  u32x4 o;
#pragma unroll
  for (int q = 0; q < 4; ++q)
    o[q] = pack2(bf2f(f2bf(lo_bf(r[q]) * rs)) * lo_bf(wv[q]), bf2f(f2bf(hi_bf(r[q]) * rs)) * hi_bf(wv[q]));
  *reinterpret_cast<u32x4*>(out + (size_t)t * H + c) = o;
}

bool launch_moe_combine_add_rmsnorm(void* out, void* residual, const void* y, const int* inv, const float* topw,
                                    const void* w, float eps, int T, int k, int H, hipStream_t st) {
  if (T == 0) return true;
  if (H % 512 || H > 8192) return false;  // whole 64-thread waves, <= 1024 threads
  moe_combine_add_rmsnorm_kernel<false><<<T, H / 8, 0, st>>>((uint16_t*)out, (uint16_t*)residual, (const uint16_t*)y,
                                                             inv, topw, (const uint16_t*)w, eps, k, H, nullptr, 0, 0);
  return true;
}

// the MoE block's tail in two launches: grouped down GEMM (its split-K partials left in the
// slab buffer) + the combine that sums them, adds into the residual and normalises.  y [R, H]
// is written only when the GEMM does not split.
bool launch_moe_down_combine_add_rmsnorm(void* out, void* residual, void* y, const void* a, const void* w2,
                                         const int* offsets, int n_groups, int R, int H, int I, int max_rows,
                                         const int* inv, const float* topw, const void* norm_w, float eps, int T,
                                         int k, hipStream_t st) {
  if (T == 0) return true;
  if (H % 512 || H > 8192) return false;
  float* ws = nullptr;
  int splits = 1;
  launch_grouped_gemm(a, w2, y, offsets, n_groups, R, H, I, max_rows, 0, st, nullptr, &ws, &splits);
  if (splits > 1)
    moe_combine_add_rmsnorm_kernel<true><<<T, H / 8, 0, st>>>((uint16_t*)out, (uint16_t*)residual, nullptr, inv, topw,
                                                              (const uint16_t*)norm_w, eps, k, H, ws, splits, R);
  else
    moe_combine_add_rmsnorm_kernel<false><<<T, H / 8, 0, st>>>((uint16_t*)out, (uint16_t*)residual, (const uint16_t*)y,
                                                               inv, topw, (const uint16_t*)norm_w, eps, k, H, nullptr, 0, 0);
  return true;
}

void launch_moe_route(float* topw, int* topi, const void* logits, int T, int E, int k,
                      hipStream_t st) {
  if (T == 0) return;
  moe_route_kernel<<<(T + 127) / 128, 128, 0, st>>>(topw, topi, (const uint16_t*)logits, T, E, k);
}

void launch_moe_permute(void* xp, int* offsets, int* src, int* inv, const void* x, const int* topi,
                        int T, int k, int H, int e0, int n_local, hipStream_t st) {
  moe_sort_kernel<<<1, 1024, 0, st>>>(offsets, src, inv, topi, T * k, e0, n_local);
  if (T * k > 0)
    moe_gather_kernel<<<T * k, 256, 0, st>>>((uint16_t*)xp, (const uint16_t*)x, src, offsets,
                                             n_local, k, H);
}

void launch_moe_combine(void* out, const void* y, const int* inv, const float* topw, int T, int k,
                        int H, hipStream_t st) {
  if (T == 0) return;
  moe_combine_kernel<<<T, 256, 0, st>>>((uint16_t*)out, (const uint16_t*)y, inv, topw, k, H);
}

}  // namespace mlop
