// Decode attention over cached latents: one query token per tile, keys and values are the SAME rows of RP
// elements (one latent head), of which the first V are values, so a step reads each latent once.
//
// A workgroup takes one tile, up to 32 heads and a partition of the keys.  Its two teams of 4 waves take
// the partition's page pairs (32 keys) in turn, each through two LDS stages (LDS-DMA, one pair ahead), and
// join at the end.  Wave w of a team works on head group w & 1 (16 heads, the MFMA columns) and half w >> 1
// of the RP dims (of an odd number of 64-dim blocks both halves hold the middle one; the second half's queries
// are zero there):
//   S^T = C . Q^T over its half, the halves' partial scores meet in LDS, both waves run the same softmax,
//   O^T += C^T . P^T for its half of the dims (with a deferred rescale).
// Every LDS row is read as K (ds_read_b128 along dims) and as V (ds_read_b64_tr_b16 along keys), so the
// image [32 keys][128 B] per 64 dims has one swizzle for both: 16-B chunk c of key t at slot c ^ sw(t),
// sw = (bit 1, bit 3, bit 2) of t, conflict-free for either kind of read.
// Key partitions leave (O, max, sum), which a second launch joins head by head (one workgroup that joined
// all of a token's heads would take longer than the attention itself).
#include <type_traits>

#include "elem.h"
#include "hybrid.h"

namespace mlop {

namespace {

constexpr int kPg = 16;
constexpr float kLow = -1.0e30f;
constexpr float kLaze = 8.f;  // deferred rescale (exp2 units)
constexpr float kLog2e = 1.4426950408889634f;
typedef short v4s16 __attribute__((ext_vector_type(4)));

// LDS reads by hand: the compiler would make every one of them wait for the LDS-DMA in flight
template <int OFF>
__device__ __forceinline__ void lds_read16(bf16x8& f, uint32_t ad) {
  asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(f) : "v"(ad), "n"(OFF));
}
template <int OFF>
__device__ __forceinline__ void lds_read_tr(v4s16& f, uint32_t ad) {
  asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(f) : "v"(ad), "n"(OFF));
}
// f(integral_constant 0), f(1), .. f(N - 1)
template <int N, int I = 0, typename F>
__device__ __forceinline__ void unrolled(F&& f) {
  if constexpr (I < N) {
    f(std::integral_constant<int, I>{});
    unrolled<N, I + 1>(f);
  }
}
// the reads older than the last `left` have arrived, a and b among them
template <typename T>
__device__ __forceinline__ void lds_wait(int left, T& a, T& b) {
  switch (left) {  // (a constant at every call)
    case 0: asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(a), "+v"(b)); break;
    case 2: asm volatile("s_waitcnt lgkmcnt(2)" : "+v"(a), "+v"(b)); break;
    case 4: asm volatile("s_waitcnt lgkmcnt(4)" : "+v"(a), "+v"(b)); break;
    default: asm volatile("s_waitcnt lgkmcnt(6)" : "+v"(a), "+v"(b)); break;
  }
}
constexpr int kAhead = 4;  // pairs of reads in flight

__device__ __forceinline__ float exp2_hw(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ int sw(int t) { return ((t & 2) << 1) | ((t >> 2) & 2) | ((t >> 2) & 1); }

}  // namespace

// NB: 64-element blocks of a latent row, NV of values (at least a.V / 64)
template <int NB, int NV>
__global__ void __launch_bounds__(512) latent_decode_kernel(AttnHdArgs a, float* __restrict__ part_o,
                                                           float* __restrict__ part_ml,
                                                           const int* __restrict__ tile_seq,
                                                           const int* __restrict__ tile_q0, int part_tokens, int nparts) {
  constexpr int RP = 64 * NB, NH = (NB + 1) / 2, NHV = (NV + 1) / 2, NK = 2 * NH, ND = 4 * NHV;
  constexpr uint32_t STAGE = NB * 4096u;  // bytes
  __shared__ __attribute__((aligned(256))) uint16_t smem[4 * STAGE / 2];  // [stage][team]; the join's exchange
  __shared__ __attribute__((aligned(16))) f32x4 sx[2][2][2][2][64];       // partial scores [team][group][half][product]
  const uint16_t* cc = reinterpret_cast<const uint16_t*>(a.k_cache);
  uint16_t* out = reinterpret_cast<uint16_t*>(a.out);
  const int tile = blockIdx.x, part = blockIdx.z, ny = gridDim.y;
  const int lane = threadIdx.x & 63, wid8 = __builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6));
  const int team = wid8 >> 2, wid = wid8 & 3;
  const int grp = wid & 1, half = wid >> 1, r = lane & 15, g4 = lane >> 4;
  const int head0 = blockIdx.y * 32 + 16 * grp, nh = min(16, a.H - head0);  // (<= 0: no such group)
  const int b0 = half * (NB - NH), v0 = half * (NV - NHV);                  // first key / value block of this half
  const int V = a.V;
  // (uniform, so that the page table is read through the scalar cache, not behind the LDS-DMA)
  const int s = __builtin_amdgcn_readfirstlane(tile_seq[tile]), qi = __builtin_amdgcn_readfirstlane(tile_q0[tile]);
  const int ql = __builtin_amdgcn_readfirstlane(a.q_len[s]), ctx = __builtin_amdgcn_readfirstlane(a.ctx_len[s]);
  const int* bt = a.bt + (size_t)s * a.bt_stride;
  const bool live = qi < ql;
  const int kv_end = live ? max(0, ctx - ql + qi + 1) : 0;
  const int k_lo = a.window > 0 ? max(0, kv_end - a.window) : 0, k_base = k_lo & ~31;
  const int p_begin = k_base + part * part_tokens;
  const int p_end = min(kv_end, p_begin + part_tokens);
  const int h_all = min(32, a.H - (int)blockIdx.y * 32);
  uint16_t* orow = out + ((size_t)tile * a.H + blockIdx.y * 32) * V;
  if (p_begin >= p_end) {  // nothing here; an empty row (graph padding) gives zeros
    if (part == 0 && kv_end <= 0 && live)
      for (int e = threadIdx.x; e < h_all * V; e += 512) orow[e] = 0;
    return;
  }

  bf16x8 qf[NK];
  {
    const bool ok = r < nh;
    const uint16_t* qrow = reinterpret_cast<const uint16_t*>(a.q) + (size_t)tile * a.q_row + (ok ? head0 + r : 0) * a.q_head +
                           b0 * 64 + g4 * 8;
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      bf16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
      if (ok && (half == 0 || b0 + (kk >> 1) >= NH)) v = *reinterpret_cast<const bf16x8*>(qrow + kk * 32);
      qf[kk] = v;
    }
  }
  f32x4 o[ND];
#pragma unroll
  for (int d = 0; d < ND; ++d) o[d] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = kLow, l = 0.f;
  const int pp0 = p_begin >> 5, pp_end = (p_end + 31) >> 5, n_pages = (p_end + kPg - 1) / kPg;
  // LDS-DMA: wave w of a team brings rows 8 w .. 8 w + 7 of every block (page A: waves 0, 1; page B: 2, 3)
  const int row32 = 8 * wid + (lane >> 3), row = row32 & 15;
  const uint32_t src_off = row * RP + (((lane & 7) ^ sw(row)) << 3);
  auto page_of = [&](int pp) {
    const auto* pages = (const __attribute__((address_space(4))) int*)(uintptr_t)bt;  // (constant: scalar loads)
    return min(max(pages[min(2 * pp + (wid >> 1), n_pages - 1)], 0), a.num_blocks - 1);
  };
  auto issue = [&](int buf, int pg) {
    uint16_t* base = smem + (2 * buf + team) * (STAGE / 2) + wid * 512;
    const uint16_t* src = cc + (size_t)pg * (kPg * RP) + src_off;
#pragma unroll
    for (int b = 0; b < NB; ++b)
      __builtin_amdgcn_global_load_lds((const void*)(src + b * 64), (lds_void_t*)(base + b * 2048), 16, 0, 0);
  };
  const uint32_t lds0 = (uint32_t)(uintptr_t)smem + team * STAGE + 4096u * b0;   // keys
  const uint32_t ldsv = (uint32_t)(uintptr_t)smem + team * STAGE + 4096u * v0;   // values
  // K: MFMA row r is key 8 (r >> 2) + (r & 3) of the pair in the first product, + 4 in the second
  const int kt = 8 * (r >> 2) + (r & 3);
  const uint32_t ka0 = lds0 + 128u * kt + 16u * (g4 ^ sw(kt & 15)), kb0 = lds0 + 128u * (kt + 4) + 16u * (g4 ^ sw((kt + 4) & 15));
  // V: transposed reads of keys 8 g4 + q (first) and + 4 (second), 16 dims at a time
  const int q = (lane >> 2) & 3, p4 = lane & 3, vt = 8 * g4 + q;
  const uint32_t va0 = ldsv + 128u * vt + 16u * ((p4 >> 1) ^ sw(vt & 15)) + 8u * (p4 & 1);
  const uint32_t vb0 = ldsv + 128u * (vt + 4) + 16u * ((p4 >> 1) ^ sw((vt + 4) & 15)) + 8u * (p4 & 1);
  const uint32_t sx_own = (uint32_t)(uintptr_t)&sx[team][grp][half][0][lane],
                 sx_other = (uint32_t)(uintptr_t)&sx[team][grp][half ^ 1][0][lane];

  if (pp0 + team < pp_end) issue(0, page_of(pp0 + team));
  int nxt = page_of(pp0 + team + 2), buf = 0;
  for (int pq = pp0; pq < pp_end; pq += 2) {
    const int pp = pq + team;
    const bool mine = pp < pp_end;  // (whole waves; every wave meets every barrier)
    wait_vmcnt<0>();
    raw_barrier();  // the pairs are in LDS for every wave; the other stage is free, and so is sx
    if (pp + 2 < pp_end) {
      issue(buf ^ 1, nxt);
      nxt = page_of(pp + 4);
    }
    const uint32_t so = buf * 2 * STAGE;
    f32x4 sa = {0.f, 0.f, 0.f, 0.f}, sb = sa;
    if (mine) {
      bf16x8 fa[kAhead], fb[kAhead];
      const uint32_t ka[2] = {ka0 + so, (ka0 ^ 64u) + so}, kb[2] = {kb0 + so, (kb0 ^ 64u) + so};
      auto rd = [&](auto kk_) {
        constexpr int kk = decltype(kk_)::value;
        lds_read16<4096 * (kk >> 1)>(fa[kk % kAhead], ka[kk & 1]);
        lds_read16<4096 * (kk >> 1)>(fb[kk % kAhead], kb[kk & 1]);
      };
      unrolled<(NK < kAhead ? NK : kAhead)>(rd);
      unrolled<NK>([&](auto kk_) {
        constexpr int kk = decltype(kk_)::value;
        lds_wait(2 * (NK - 1 - kk < kAhead - 1 ? NK - 1 - kk : kAhead - 1), fa[kk % kAhead], fb[kk % kAhead]);
        sa = mfma16(fa[kk % kAhead], qf[kk], sa);
        sb = mfma16(fb[kk % kAhead], qf[kk], sb);
        if constexpr (kk + kAhead < NK) rd(std::integral_constant<int, kk + kAhead>{});
      });
      asm volatile("ds_write_b128 %0, %1\n\tds_write_b128 %0, %2 offset:1024" ::"v"(sx_own), "v"(sa), "v"(sb) : "memory");
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    raw_barrier();
    if (mine) {
      {
        f32x4 ta, tb;
        asm volatile("ds_read_b128 %0, %2\n\tds_read_b128 %1, %2 offset:1024\n\ts_waitcnt lgkmcnt(0)"
                     : "=&v"(ta), "=&v"(tb)
                     : "v"(sx_other)
                     : "memory");
        sa += ta;
        sb += tb;
      }
      const int tokA = pp * 32 + g4 * 8, tokB = tokA + 4;
      float pa[4], pb[4], mx = kLow;
#pragma unroll
      for (int i = 0; i < 4; ++i) pa[i] = sa[i] * a.scale_log2, pb[i] = sb[i] * a.scale_log2;
      if (pp * 32 + 31 >= p_end || pp * 32 < k_lo) {
        asm volatile("");  // keep the branch: the mask is needed at the range's ends only
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          pa[i] = tokA + i < p_end && tokA + i >= k_lo ? pa[i] : -INFINITY;
          pb[i] = tokB + i < p_end && tokB + i >= k_lo ? pb[i] : -INFINITY;
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) mx = fmaxf(mx, fmaxf(pa[i], pb[i]));
      mx = max_x16_x32(mx);
      if (__ballot(mx - m > kLaze)) {
        const float m_new = fmaxf(m, mx), alpha = exp2_hw(m - m_new);
        m = m_new;
        l *= alpha;
#pragma unroll
        for (int d = 0; d < ND; ++d) o[d] *= alpha;
      }
      u32x4 pw;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        pa[i] = exp2_hw(pa[i] - m);
        pb[i] = exp2_hw(pb[i] - m);
        l += pa[i] + pb[i];
      }
      pw = u32x4{pack2(pa[0], pa[1]), pack2(pa[2], pa[3]), pack2(pb[0], pb[1]), pack2(pb[2], pb[3])};
      const bf16x8 pf = __builtin_bit_cast(bf16x8, pw);
      v4s16 lo[kAhead], hi[kAhead];
      uint32_t va[4], vb[4];
#pragma unroll
      for (int x = 0; x < 4; ++x) va[x] = (va0 ^ (32u * x)) + so, vb[x] = (vb0 ^ (32u * x)) + so;
      auto rd = [&](auto d_) {
        constexpr int d = decltype(d_)::value;
        lds_read_tr<4096 * (d >> 2)>(lo[d % kAhead], va[d & 3]);
        lds_read_tr<4096 * (d >> 2)>(hi[d % kAhead], vb[d & 3]);
      };
      unrolled<kAhead>(rd);
      unrolled<ND>([&](auto d_) {
        constexpr int d = decltype(d_)::value;
        lds_wait(2 * (ND - 1 - d < kAhead - 1 ? ND - 1 - d : kAhead - 1), lo[d % kAhead], hi[d % kAhead]);
        bf16x8 f;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          f[e] = lo[d % kAhead][e];
          f[4 + e] = hi[d % kAhead][e];
        }
        o[d] = mfma16(f, pf, o[d]);
        if constexpr (d + kAhead < ND) rd(std::integral_constant<int, d + kAhead>{});
      });
    }
    buf ^= 1;
  }
  l = sum_x16_x32(l);
  {  // the second team's result joins the first's
    __syncthreads();
    f32x4* xo = reinterpret_cast<f32x4*>(smem) + (size_t)wid * ND * 64 + lane;
    float* xm = reinterpret_cast<float*>(sx) + wid * 128 + lane * 2;
    if (team == 1) {
#pragma unroll
      for (int d = 0; d < ND; ++d) xo[d * 64] = o[d];
      xm[0] = m;
      xm[1] = l;
    }
    __syncthreads();
    if (team == 1) return;
    const float m1 = xm[0], l1 = xm[1], M = fmaxf(m, m1), f0 = exp2_hw(m - M), f1 = exp2_hw(m1 - M);
    m = M;
    l = l * f0 + l1 * f1;
#pragma unroll
    for (int d = 0; d < ND; ++d) o[d] = o[d] * f0 + xo[d * 64] * f1;
  }
  const bool ok = r < nh;
  // 64-dim block v0 + i of the values is this wave's to store
  auto mine_v = [&](int i) { return (half == 0 || v0 + i >= NHV) && (v0 + i) * 64 < V; };
  const size_t slab = (((size_t)tile * ny + blockIdx.y) * 2 + grp) * nparts;  // 16 heads each
  if (nparts == 1) {
    float L = l, f = 1.f;
    if (a.sink && ok) {
      const float s2 = a.sink[head0 + r] * kLog2e, M = fmaxf(m, s2);
      f = exp2f(m - M);
      L = l * f + exp2f(s2 - M);
    }
    const float inv = L > 0.f ? f / L : 0.f;
    if (ok) {
#pragma unroll
      for (int d = 0; d < ND; ++d)
        if (mine_v(d >> 2)) {
          const float v[4] = {o[d][0] * inv, o[d][1] * inv, o[d][2] * inv, o[d][3] * inv};
          stn<4>(orow + (size_t)(16 * grp + r) * V + v0 * 64 + 16 * d + 4 * g4, v);
        }
    }
    return;
  }
  // partial (O, m, l) of this key range
  if (ok) {
    float* po = part_o + ((slab + part) * 16 + r) * V + v0 * 64 + 4 * g4;
#pragma unroll
    for (int d = 0; d < ND; ++d)
      if (mine_v(d >> 2)) *reinterpret_cast<f32x4*>(po + 16 * d) = o[d];
    if (half == 0 && g4 == 0) {
      float* ml = part_ml + ((slab + part) * 16 + r) * 2;
      ml[0] = m;
      ml[1] = l;
    }
  }
}

// the partitions of one (tile, head): 4 elements per thread
__global__ void __launch_bounds__(192) latent_combine_kernel(AttnHdArgs a, const float* __restrict__ part_o,
                                                             const float* __restrict__ part_ml,
                                                             const int* __restrict__ tile_seq,
                                                             const int* __restrict__ tile_q0, int part_tokens, int nparts) {
  const int tile = blockIdx.x, head = blockIdx.y, c = threadIdx.x * 4, V = a.V;
  const int s = tile_seq[tile], qi = tile_q0[tile], ql = a.q_len[s], ctx = a.ctx_len[s];
  const int kv_end = qi < ql ? max(0, ctx - ql + qi + 1) : 0;
  if (kv_end == 0 || c >= V) return;  // (an empty row was zeroed)
  const int k_base = (a.window > 0 ? max(0, kv_end - a.window) : 0) & ~31;
  const int nvalid = min(nparts, (kv_end - k_base + part_tokens - 1) / part_tokens);
  const size_t slab = ((size_t)tile * (cdiv(a.H, 32) * 2) + (head >> 4)) * nparts * 16 + (head & 15);
  const float* ml = part_ml + slab * 2;
  const float* po = part_o + slab * V + c;
  const float s2 = a.sink ? a.sink[head] * kLog2e : kLow;
  float M = s2;
  for (int p = 0; p < nvalid; ++p) M = fmaxf(M, ml[p * 32]);
  float L = a.sink ? exp2f(s2 - M) : 0.f;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int p = 0; p < nvalid; ++p) {
    const float f = exp2f(ml[p * 32] - M);
    L += f * ml[p * 32 + 1];
    acc += f * *reinterpret_cast<const f32x4*>(po + (size_t)p * 16 * V);
  }
  const float inv = L > 0.f ? 1.f / L : 0.f;
  const float v[4] = {acc[0] * inv, acc[1] * inv, acc[2] * inv, acc[3] * inv};
  stn<4>(reinterpret_cast<uint16_t*>(a.out) + ((size_t)tile * a.H + head) * V + c, v);
}

void launch_latent_decode(const AttnHdArgs& a, float* part_o, float* part_ml, const int* tile_seq,
                          const int* tile_q0, int num_tiles, int part_tokens, int nparts, hipStream_t st) {
  const dim3 grid(num_tiles, cdiv(a.H, 32), nparts);
#define MLOP_LD_V(N, V) \
  latent_decode_kernel<N, V><<<grid, 512, 0, st>>>(a, part_o, part_ml, tile_seq, tile_q0, part_tokens, nparts)
#define MLOP_LD(N)                                                        \
  case N:                                                                 \
    if (N > 1 && a.V / 64 < N) MLOP_LD_V(N, (N > 1 ? N - 1 : 1));         \
    else MLOP_LD_V(N, N);                                                 \
    break;
  switch (a.KP / 64) {
    MLOP_LD(1) MLOP_LD(2) MLOP_LD(3) MLOP_LD(4) MLOP_LD(5) MLOP_LD(6) MLOP_LD(7) MLOP_LD(8) MLOP_LD(9)
    default: break;
  }
#undef MLOP_LD
#undef MLOP_LD_V
  if (nparts > 1)
    latent_combine_kernel<<<dim3(num_tiles, a.H), cdiv(a.V, 256) * 64, 0, st>>>(a, part_o, part_ml, tile_seq, tile_q0,
                                                                                part_tokens, nparts);
}

}  // namespace mlop
