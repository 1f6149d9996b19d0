// Paged attention of any head sizes (query / key size D, value size V, any GQA ratio) with a
// softmax sink, a score scale and a per-head output gate, beside attention.hip's kernels (head
// size 128 for keys and values, power-of-two groups).  Differences that matter here:
//
//   * cache rows are padded to 64 elements (KP, VP = 64 NKB, 64 NVB): a row is whole 128-B lines
//     and every LDS image is made of [32 keys][128 B] blocks with one swizzle, whatever the sizes:
//       K block: 16-B chunk c of key k at slot c ^ ((k >> 1) & 7)     (ds_read_b128)
//       V block: chunk c of key k at slot c ^ vsw(k)                   (ds_read_b64_tr_b16)
//     both conflict-free for the fragment reads;
//   * the query tile does not depend on the GQA ratio (layers of one model may differ in it): a
//     decode tile is one token with up to 16 heads of a kv head as MFMA rows (more heads take
//     further workgroups), a prompt tile is 128 tokens of ONE head;
//   * sink: a number per head that joins the softmax's denominator once, with no key and no value;
//   * gate: head h's output times sigmoid(gate[t, h]), or an element's with its own gate, in the epilogue;
//   * window: a token sees itself and the window - 1 tokens before it; pages in front are not read;
//   * a prompt's keys and values may also come from dense rows (latent attention's expanded keys);
//   * rot: a part of a prompt's query heads may turn by the position as it is read.
// The sizes above 256 and fp32 operands take attn_any_kernel (one wave per query and head).
//
// REQUIREMENT: the cache is zero-initialised at allocation (as attention.hip's) and the pad
// elements are never written.
#include "elem.h"
#include "hybrid.h"

namespace mlop {

namespace {

constexpr int kPg = 16;  // tokens per page
constexpr float kLow = -1.0e30f;
constexpr float kLog2e = 1.4426950408889634f;
constexpr float kLaze = 8.f;  // deferred rescale of the prompt kernel (exp2 units)

using f32x16 = __attribute__((ext_vector_type(16))) float;
typedef short v4s16 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) v4s16 lds_v4s16;

__device__ __forceinline__ float exp2_hw(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ int vsw(int t) { return ((t & 2) << 1) | ((t >> 2) & 2); }
__device__ __forceinline__ f32x16 mfma32b(bf16x8 a, bf16x8 b, f32x16 c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ uint32_t pk_bf16(float lo, float hi) {
  uint32_t r;
  asm("v_cvt_pk_bf16_f32 %0, %1, %2" : "=v"(r) : "v"(lo), "v"(hi));
  return r;
}
__device__ __forceinline__ float gate_of(const AttnHdArgs& a, int tok, int head) {
  if (!a.gate || a.gate_elem) return 1.f;
  const float g = bf2f(reinterpret_cast<const uint16_t*>(a.gate)[(size_t)tok * a.gate_stride + head]);
  return 1.f / (1.f + __expf(-g));
}

// dims c .. c + 7 of a query head, the rotated ones among them turned by position p
__device__ __forceinline__ bf16x8 turn8(const AttnHdArgs& a, bf16x8 x, int c, int p) {
  const int d0 = c - a.rot_lo, half = a.n_rot >> 1;
  if (d0 + 8 <= 0 || d0 >= a.n_rot) return x;
  const float* cs = a.rot + (size_t)min(max(p, 0), a.n_pos - 1) * a.n_rot;
#pragma unroll
  for (int e = 0; e < 8; e += 2) {
    if (d0 + e < 0 || d0 + e >= a.n_rot) continue;
    const float co = cs[(d0 + e) >> 1], si = cs[half + ((d0 + e) >> 1)];
    const float u = bf2f_s(x[e]), v = bf2f_s(x[e + 1]);
    x[e] = (short)f2bf(u * co - v * si);
    x[e + 1] = (short)f2bf(v * co + u * si);
  }
  return x;
}

// an element's own gate
__device__ __forceinline__ float gate_at(const AttnHdArgs& a, int tok, int head, int c) {
  const float g = bf2f(reinterpret_cast<const uint16_t*>(a.gate)[(size_t)tok * a.gate_stride + head * a.V + c]);
  return 1.f / (1.f + __expf(-g));
}
template <int N>
__device__ __forceinline__ void gate_elems(const AttnHdArgs& a, int tok, int head, int c, float (&v)[N]) {
  if (!a.gate || !a.gate_elem) return;
  if (a.gate_vec) {  // V a multiple of 4
    const uint16_t* g = reinterpret_cast<const uint16_t*>(a.gate) + (size_t)tok * a.gate_stride + head * a.V + c;
#pragma unroll
    for (int j = 0; j < N; j += 4) {
      if (c + j >= a.V) continue;
      float z[4];
      ldn<4>(g + j, z);
#pragma unroll
      for (int i = 0; i < 4; ++i) v[j + i] *= __builtin_amdgcn_rcpf(1.f + __expf(-z[i]));
    }
    return;
  }
#pragma unroll
  for (int j = 0; j < N; ++j)
    if (c + j < a.V) v[j] *= gate_at(a, tok, head, c + j);
}

// 8 consecutive outputs of a head, dims c .. c + 7 (only those below V)
__device__ __forceinline__ void store8(uint16_t* dst, int c, int V, const float (&v)[8]) {
  if (V % 8 == 0) {
    if (c < V) stn<8>(dst + c, v);
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (c + j < V) dst[c + j] = f2bf(v[j]);
  }
}

}  // namespace

// Decode: one (tile = one query token, kv head, 16-head group, key partition) per workgroup, page
// pairs (32 keys) round-robin over its 4 waves; attention.hip's paged_attn_kernel with the
// products S^T = K . Q^T and O^T = V^T . P^T.
template <int NKB, int NVB>
__global__ void __launch_bounds__(256) paged_hd_kernel(AttnHdArgs a, float* __restrict__ part_o,
                                                       float* __restrict__ part_ml, int* __restrict__ sem,
                                                       const int* __restrict__ tile_seq,
                                                       const int* __restrict__ tile_q0, int part_tokens, int nparts) {
  constexpr int KP = 64 * NKB, VP = 64 * NVB, NK = 2 * NKB, ND = 4 * NVB;
  // wave w's V image (NVB blocks of 4 KB) lies inside sm_o[w], which it alone writes after its loop
  __shared__ __attribute__((aligned(256))) float sm_o[4][16][VP + 4];
  __shared__ float sm_m[4][16];
  __shared__ float sm_l[4][16];
  __shared__ int sm_last;

  const uint16_t* kc = reinterpret_cast<const uint16_t*>(a.k_cache);
  const uint16_t* vc = reinterpret_cast<const uint16_t*>(a.v_cache);
  uint16_t* out = reinterpret_cast<uint16_t*>(a.out);
  const int Gq = a.H / a.G, hg = cdiv(Gq, 16);
  const int tile = blockIdx.x, part = blockIdx.z, ny = gridDim.y;
  const int kvh = blockIdx.y / hg, h0 = (blockIdx.y % hg) * 16, nh = min(16, Gq - h0), head0 = kvh * Gq + h0;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int s = tile_seq[tile], qi = tile_q0[tile];
  const int ql = a.q_len[s], ctx = a.ctx_len[s], tok = a.q_start[s] + qi;
  const int* bt = a.bt + (size_t)s * a.bt_stride;
  const bool live = qi < ql;
  const int kv_end = live ? max(0, ctx - ql + qi + 1) : 0;
  const int orow = a.by_tile ? tile : tok;  // row of q and out
  // keys [k_lo, kv_end) in partitions counted from k_lo's page pair
  const int k_lo = a.window > 0 ? max(0, kv_end - a.window) : 0, k_base = k_lo & ~31;
  const int p_begin = k_base + part * part_tokens;
  const int p_end = min(kv_end, p_begin + part_tokens);
  if (p_begin >= p_end && nparts > 1) {
    // no partition of an empty row (graph padding) draws the last ticket: partition 0 zeroes it
    if (part == 0 && kv_end <= 0 && live) {
      for (int e = threadIdx.x; e < nh * a.V; e += 256)
        out[(size_t)orow * a.out_row + (head0 + e / a.V) * a.V + e % a.V] = 0;
    }
    return;
  }

  const int r = lane & 15, g4 = lane >> 4;
  const bool row_ok = live && r < nh;
  bf16x8 qf[NK];
  {
    const uint16_t* qrow = reinterpret_cast<const uint16_t*>(a.q) + (size_t)orow * a.q_row + (head0 + (row_ok ? r : 0)) * a.q_head;
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      const bf16x8 v = live ? *reinterpret_cast<const bf16x8*>(qrow + kk * 32 + g4 * 8) : bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
      qf[kk] = row_ok ? v : bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
    }
  }
  f32x4 o[ND];
#pragma unroll
  for (int d = 0; d < ND; ++d) o[d] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = kLow, l = 0.f;
  const int pp_begin = p_begin >> 5, pp_end = (p_end + 31) >> 5;
  const int n_pages = (p_end + kPg - 1) / kPg;
  const size_t k_page = (size_t)a.G * kPg * KP, v_page = (size_t)a.G * kPg * VP;
  const size_t k_head = (size_t)kvh * kPg * KP, v_head = (size_t)kvh * kPg * VP;
  const uint32_t vimg = (uint32_t)(uintptr_t)&sm_o[wid][0][0];
  auto page_at = [&](int i) { return min(max(bt[i], 0), a.num_blocks - 1); };  // never out of the pool
  uint32_t vb0;
  {
    const int q = (lane >> 2) & 3, p = lane & 3, row = 8 * g4 + q;
    vb0 = vimg + 128u * row + 16u * ((p >> 1) ^ vsw(row & 15)) + 8u * (p & 1);
  }
  int pgA = 0, pgB = 0;
  if (pp_begin + wid < pp_end) {
    pgA = page_at(2 * (pp_begin + wid));
    pgB = 2 * (pp_begin + wid) + 1 < n_pages ? page_at(2 * (pp_begin + wid) + 1) : pgA;
  }
  for (int pp = pp_begin + wid; pp < pp_end; pp += 4) {
    // K rows of MFMA row r: pair tokens 8 (r >> 2) + (r & 3) (first product) and + 4 (second)
    const uint16_t* kR = kc + (r >> 3 ? pgB : pgA) * k_page + k_head + (8 * ((r >> 2) & 1) + (r & 3)) * KP;
    bf16x8 ka[NK], kb[NK];
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      ka[kk] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(kR + kk * 32 + g4 * 8));
      kb[kk] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(kR + 4 * KP + kk * 32 + g4 * 8));
    }
    // the pair's V image by LDS-DMA (1 KB = 8 rows of a block each), behind the K loads
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
    for (int b = 0; b < NVB; ++b)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int row = (8 * i + (lane >> 3)) & 15;
        const uint16_t* src = vc + (i < 2 ? pgA : pgB) * v_page + v_head + row * VP + b * 64 + (((lane & 7) ^ vsw(row)) << 3);
        __builtin_amdgcn_global_load_lds((const void*)src, (lds_void_t*)(uintptr_t)(vimg + 4096u * b + 1024u * i), 16, 0,
                                         2 /* nt */);
      }
    if (pp + 4 < pp_end) {
      pgA = page_at(2 * (pp + 4));
      pgB = 2 * (pp + 4) + 1 < n_pages ? page_at(2 * (pp + 4) + 1) : pgA;
    }
    f32x4 sa = {0.f, 0.f, 0.f, 0.f}, sb = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      sa = mfma16(ka[kk], qf[kk], sa);
      sb = mfma16(kb[kk], qf[kk], sb);
    }
    const int tokA = pp * 32 + g4 * 8, tokB = tokA + 4;
    float pa[4], pb[4], mx = kLow;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      pa[i] = tokA + i < p_end && tokA + i >= k_lo ? sa[i] * a.scale_log2 : -INFINITY;
      pb[i] = tokB + i < p_end && tokB + i >= k_lo ? sb[i] * a.scale_log2 : -INFINITY;
      mx = fmaxf(mx, fmaxf(pa[i], pb[i]));
    }
    mx = max_x16_x32(mx);
    const float m_new = fmaxf(m, mx), alpha = exp2_hw(m - m_new);
    m = m_new;
    float rs = 0.f;
    bf16x8 pf;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      pa[i] = exp2_hw(pa[i] - m_new);
      pb[i] = exp2_hw(pb[i] - m_new);
      rs += pa[i] + pb[i];
      pf[i] = (short)f2bf(pa[i]);
      pf[4 + i] = (short)f2bf(pb[i]);
    }
    l = l * alpha + rs;
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // this wave's V image has landed
    uint32_t vb = vb0;
    asm volatile("" : "+v"(vb));
#pragma unroll
    for (int d = 0; d < ND; ++d) {
      const uint32_t ad = (vb ^ (32u * (d & 3))) + 4096u * (d >> 2);
      const v4s16 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s16*)(uintptr_t)ad);
      const v4s16 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s16*)(uintptr_t)(ad + 512u));
      bf16x8 f;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        f[e] = lo[e];
        f[4 + e] = hi[e];
      }
      o[d] *= alpha;
      o[d] = mfma16(f, pf, o[d]);
    }
  }

  l = sum_x16_x32(l);
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // the last image is read before sm_o overwrites it
#pragma unroll
  for (int d = 0; d < ND; ++d)
#pragma unroll
    for (int i = 0; i < 4; ++i) sm_o[wid][r][d * 16 + g4 * 4 + i] = o[d][i];
  if (g4 == 0) {
    sm_m[wid][r] = m;
    sm_l[wid][r] = l;
  }
  __syncthreads();

  constexpr int CH = VP / 8;  // 8-element column groups of a row
  const size_t slab0 = ((size_t)tile * ny + blockIdx.y) * nparts;
  for (int e = threadIdx.x; e < 16 * CH; e += 256) {
    const int rr = e / CH, c = (e % CH) * 8;
    if (rr >= nh || !live) continue;
    float M = kLow;
#pragma unroll
    for (int w = 0; w < 4; ++w) M = fmaxf(M, sm_m[w][rr]);
    if (nparts == 1 && a.sink) M = fmaxf(M, a.sink[head0 + rr] * kLog2e);
    float L = 0.f, acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float f = exp2f(sm_m[w][rr] - M);
      L += f * sm_l[w][rr];
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[j] += f * sm_o[w][rr][c + j];
    }
    if (nparts == 1) {
      if (a.sink) L += exp2f(a.sink[head0 + rr] * kLog2e - M);
      const float inv = L > 0.f ? gate_of(a, tok, head0 + rr) / L : 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[j] *= inv;
      gate_elems(a, tok, head0 + rr, c, acc);
      store8(out + (size_t)orow * a.out_row + (head0 + rr) * a.V, c, a.V, acc);
    } else {
      // partial (O, m, l) of this key range, stored through to the memory side (sc1) so that the
      // ticket below needs no release fence
      const size_t slab = (slab0 + part) * 16;
      const auto rs_o = __builtin_amdgcn_make_buffer_rsrc(part_o + slab * VP, 0, 16 * VP * 4, 0x00020000);
      const uint32_t oo = (uint32_t)(rr * VP + c) * 4u;
      u32x4 w0, w1;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        w0[j] = __float_as_uint(acc[j]);
        w1[j] = __float_as_uint(acc[4 + j]);
      }
      __builtin_amdgcn_raw_buffer_store_b128(w0, rs_o, oo, 0, 16 /* sc1 */);
      __builtin_amdgcn_raw_buffer_store_b128(w1, rs_o, oo + 16u, 0, 16 /* sc1 */);
      if (c == 0) {
        const auto rs_ml = __builtin_amdgcn_make_buffer_rsrc(part_ml + slab * 2, 0, 16 * 2 * 4, 0x00020000);
        __builtin_amdgcn_raw_buffer_store_b32(__float_as_uint(M), rs_ml, (uint32_t)rr * 8u, 0, 16);
        __builtin_amdgcn_raw_buffer_store_b32(__float_as_uint(L), rs_ml, (uint32_t)rr * 8u + 4u, 0, 16);
      }
    }
  }
  if (nparts == 1) return;
  // the partition that draws the last ticket combines all of them and re-arms the counter
  // (attention.hip's hand-off: sc1 stores, vmcnt(0) in every wave, barrier, relaxed ticket,
  // agent acquire on the consumer's side)
  const int nvalid = min(nparts, (kv_end - k_base + part_tokens - 1) / part_tokens);
  int* cnt = sem + (size_t)tile * ny + blockIdx.y;
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  if (threadIdx.x == 0) {
    const int t = __hip_atomic_fetch_add(cnt, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    sm_last = (t == nvalid - 1);
  }
  __syncthreads();
  if (!sm_last) return;
  if (threadIdx.x == 0) {
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "agent");
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __hip_atomic_store(cnt, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  }
  __syncthreads();
  for (int e = threadIdx.x; e < 16 * CH; e += 256) {
    const int rr = e / CH, c = (e % CH) * 8;
    if (rr >= nh || !live) continue;
    float M = a.sink ? a.sink[head0 + rr] * kLog2e : kLow;
    for (int p = 0; p < nvalid; ++p) M = fmaxf(M, part_ml[((slab0 + p) * 16 + rr) * 2]);
    float L = a.sink ? exp2f(a.sink[head0 + rr] * kLog2e - M) : 0.f;
    float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    for (int p = 0; p < nvalid; ++p) {
      const size_t pb = (slab0 + p) * 16 + rr;
      const float f = exp2f(part_ml[pb * 2] - M);
      L += f * part_ml[pb * 2 + 1];
      float v[8];
      ldn<8>(part_o + pb * VP + c, v);
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[j] += f * v[j];
    }
    const float inv = L > 0.f ? gate_of(a, tok, head0 + rr) / L : 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[j] *= inv;
    gate_elems(a, tok, head0 + rr, c, acc);
    store8(out + (size_t)orow * a.out_row + (head0 + rr) * a.V, c, a.V, acc);
  }
}

// Prompt chunks: 128 query tokens of one head per workgroup against their whole causal range,
// attention.hip's flash32 scheme (32x32x16 MFMA, softmax on the lane, 3-deep LDS-DMA ring of page
// pairs, counted vmcnt, one raw barrier per pair, deferred rescale).
template <int NKB, int NVB>
__global__ void __launch_bounds__(256, (NKB + NVB) <= 5 ? 2 : 1) flash_hd_kernel(AttnHdArgs a,
                                                                                const int* __restrict__ ptile_seq,
                                                                                const int* __restrict__ ptile_q0) {
  constexpr int KP = 64 * NKB, VP = 64 * NVB, NQ = 4 * NKB, ND = 2 * NVB;
  constexpr uint32_t STAGE = (NKB + NVB) * 4096u;  // bytes: NKB K blocks, NVB V blocks
  constexpr int OPS = NKB + NVB;                   // LDS-DMAs of a wave per pair
  constexpr int STAGES = 3;
  __shared__ __attribute__((aligned(256))) uint16_t smem[STAGES * STAGE / 2];
  const uint16_t* kc = reinterpret_cast<const uint16_t*>(a.k_cache);
  const uint16_t* vc = reinterpret_cast<const uint16_t*>(a.v_cache);
  const int lane = threadIdx.x & 63, wid = __builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6));
  // kv head fastest over the grid: a kv head's workgroups share an XCD's L2
  const int Gq = a.H / a.G;
  const int kvh = blockIdx.x % a.G, rest = blockIdx.x / a.G, head = kvh * Gq + rest % Gq, tile = rest / Gq;
  const int s = ptile_seq[tile], q0 = ptile_q0[tile];
  const int ql = a.q_len[s], ctx = a.ctx_len[s], qs = a.q_start[s];
  const int last_q = min(q0 + kHdTile, ql) - 1;
  const int kv_end = ctx - ql + last_q + 1;
  const int n_pairs = (kv_end + 31) >> 5;
  const int pp0 = a.window > 0 ? max(0, ctx - ql + q0 - a.window + 1) >> 5 : 0;  // first pair a query sees
  const int n_pages = (kv_end + kPg - 1) / kPg;
  const int col = lane & 31, h = lane >> 5;
  const int qi = q0 + 32 * wid + col;
  const bool q_ok = qi < ql;
  const int pos_r = q_ok ? ctx - ql + qi : -1;
  const int low_r = a.window > 0 ? pos_r - a.window + 1 : 0;  // first key of this row
  // positions of this wave's rows: pairs past the last are masked whole, pairs up to the first need no mask
  const bool wave_live = q0 + 32 * wid < ql;
  const int wave_min = ctx - ql + q0 + 32 * wid, wave_max = min(wave_min + 31, kv_end - 1);
  // first key any row of the wave sees, first key all of them see
  const int wave_low = a.window > 0 ? wave_min - a.window + 1 : 0, wave_in = a.window > 0 ? wave_max - a.window + 1 : 0;

  bf16x8 qf[NQ];
  {
    const uint16_t* qrow = reinterpret_cast<const uint16_t*>(a.q) + (size_t)(qs + (q_ok ? qi : 0)) * a.q_row + head * a.q_head + 8 * h;
#pragma unroll
    for (int t = 0; t < NQ; ++t) {
      bf16x8 v = *reinterpret_cast<const bf16x8*>(qrow + 16 * t);
      if (a.rot) v = turn8(a, v, 16 * t + 8 * h, pos_r);
      qf[t] = q_ok ? v : bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
    }
  }
  f32x16 o[ND];
#pragma unroll
  for (int d = 0; d < ND; ++d)
#pragma unroll
    for (int e = 0; e < 16; ++e) o[d][e] = 0.f;
  float m = kLow, l = 0.f;

  const int* bt = a.bt + (size_t)s * a.bt_stride;
  const int xb = a.xbase ? a.xbase[s] : 0;
  // LDS-DMA: wave w brings rows 8w .. 8w + 7 of every block (page A: waves 0, 1; page B: 2, 3)
  const int row32 = 8 * wid + (lane >> 3), row = row32 & 15;
  const size_t k_off = kvh * a.k_head + row * a.k_row + (((lane & 7) ^ ((row32 >> 1) & 7)) << 3);
  const size_t v_off = kvh * a.v_head + row * a.v_row + (((lane & 7) ^ vsw(row)) << 3);
  auto page_of = [&](int pair) {  // first row of this wave's page
    const int i = min(2 * pair + (wid >> 1), n_pages - 1);
    return a.xbase ? xb + i * kPg : min(max(bt[i], 0), a.num_blocks - 1) * kPg;
  };
  auto issue = [&](int buf, int pg) {
    uint16_t* base = smem + buf * (STAGE / 2) + wid * 512;
    const uint16_t* ks = kc + pg * a.k_pitch + k_off;
    const uint16_t* vs = vc + pg * a.v_pitch + v_off;
#pragma unroll
    for (int b = 0; b < NKB; ++b)
      __builtin_amdgcn_global_load_lds((const void*)(ks + b * 64), (lds_void_t*)(base + b * 2048), 16, 0, 0);
#pragma unroll
    for (int b = 0; b < NVB; ++b)
      __builtin_amdgcn_global_load_lds((const void*)(vs + b * 64), (lds_void_t*)(base + (NKB + b) * 2048), 16, 0, 0);
  };
  const uint32_t lds0 = (uint32_t)(uintptr_t)smem;
  const uint32_t k_b0 = lds0 + 128u * col + 16u * (h ^ ((col >> 1) & 7));
  uint32_t v_b0;
  {
    const int g = lane >> 4, q = (lane >> 2) & 3, p = lane & 3, t = 4 * h + q;
    v_b0 = lds0 + NKB * 4096u + 128u * t + 16u * ((2 * (g & 1) + (p >> 1)) ^ vsw(t)) + 8u * (p & 1);
  }

  // S^T of the pair in ring slot at byte offset so: K fragment t = keys, dims 16t + 8h .. + 7
  auto qk = [&](uint32_t so) {
    uint32_t kb = k_b0 + so;
    asm volatile("" : "+v"(kb));
    f32x16 sc;
#pragma unroll
    for (int e = 0; e < 16; ++e) sc[e] = 0.f;
    bf16x8 kf[4];
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#define MLOP_KREAD(t, f)                                                                                       \
  asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(f) : "v"(kb ^ (32u * ((t) & 3))), "n"(4096 * ((t) >> 2)))
    MLOP_KREAD(0, kf[0]);
    MLOP_KREAD(1, kf[1]);
    MLOP_KREAD(2, kf[2]);
    MLOP_KREAD(3, kf[3]);
#pragma unroll
    for (int t = 0; t < NQ; ++t) {
      bf16x8& f = kf[t & 3];
      if (t <= NQ - 4) asm volatile("s_waitcnt lgkmcnt(3)" : "+v"(f));
      else if (t == NQ - 3) asm volatile("s_waitcnt lgkmcnt(2)" : "+v"(f));
      else if (t == NQ - 2) asm volatile("s_waitcnt lgkmcnt(1)" : "+v"(f));
      else asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(f));
      sc = mfma32b(f, qf[t], sc);
      if (t + 4 < NQ) {
        uint32_t ad = kb ^ (32u * (t & 3));
        switch ((t + 4) >> 2) {
          case 1: asm volatile("ds_read_b128 %0, %1 offset:4096" : "=v"(f) : "v"(ad)); break;
          case 2: asm volatile("ds_read_b128 %0, %1 offset:8192" : "=v"(f) : "v"(ad)); break;
          default: asm volatile("ds_read_b128 %0, %1 offset:12288" : "=v"(f) : "v"(ad)); break;
        }
      }
    }
#undef MLOP_KREAD
    return sc;
  };
  auto softmax = [&](f32x16 sc, int pp, bf16x8 (&pf)[2]) {
    if (pp * 32 + 31 > wave_min || pp * 32 < wave_in) {
      asm volatile("");  // keep the branch: the mask is needed on the diagonal and at the window's edge only
#pragma unroll
      for (int e = 0; e < 16; ++e) {
        const int tk = pp * 32 + (e & 3) + 8 * (e >> 2) + 4 * h;
        sc[e] = tk <= pos_r && tk >= low_r ? sc[e] : -INFINITY;
      }
    }
    float mx = fmaxf(fmaxf(sc[0], sc[1]), sc[2]);
#pragma unroll
    for (int e = 3; e < 15; e += 2) mx = fmaxf(fmaxf(mx, sc[e]), sc[e + 1]);
    mx = fmaxf(mx, sc[15]);
    {
      const auto sw = __builtin_amdgcn_permlane32_swap(__float_as_uint(mx), __float_as_uint(mx), false, false);
      mx = fmaxf(__uint_as_float(sw[0]), __uint_as_float(sw[1]));
    }
    if (__ballot((mx - m) * a.scale_log2 > kLaze)) {
      const float m_new = fmaxf(m, mx), alpha = exp2_hw((m - m_new) * a.scale_log2);
      m = m_new;
#pragma unroll
      for (int d = 0; d < ND; ++d) o[d] *= alpha;
      l *= alpha;
    }
    const float mc = -m * a.scale_log2;
    float rs = 0.f;
    u32x4 w[2];
#pragma unroll
    for (int e = 0; e < 16; e += 2) {
      const float p0 = exp2_hw(fmaf(sc[e], a.scale_log2, mc)), p1 = exp2_hw(fmaf(sc[e + 1], a.scale_log2, mc));
      rs += p0 + p1;
      w[e >> 3][(e & 7) >> 1] = pk_bf16(p0, p1);
    }
    pf[0] = __builtin_bit_cast(bf16x8, w[0]);
    pf[1] = __builtin_bit_cast(bf16x8, w[1]);
    l += rs;
  };
  auto pv = [&](uint32_t so, const bf16x8 (&pf)[2]) {
    uint32_t vb = v_b0 + so;
    asm volatile("" : "+v"(vb));
    // 32-dim block d: rows of page A (two transposed reads) and of page B
    auto rd = [&](int d, v4s16 (&x)[4]) {
      const uint32_t a0 = (vb ^ (64u * (d & 1))) + 4096u * (d >> 1), a1 = a0 ^ 32u;
      asm volatile(
          "ds_read_b64_tr_b16 %0, %4\n"
          "ds_read_b64_tr_b16 %1, %5 offset:1024\n"
          "ds_read_b64_tr_b16 %2, %4 offset:2048\n"
          "ds_read_b64_tr_b16 %3, %5 offset:3072\n"
          : "=&v"(x[0]), "=&v"(x[1]), "=&v"(x[2]), "=&v"(x[3])
          : "v"(a0), "v"(a1));
    };
    auto frag = [&](const v4s16& lo, const v4s16& hi) {
      bf16x8 f;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        f[e] = lo[e];
        f[4 + e] = hi[e];
      }
      return f;
    };
    v4s16 ra[4], rb[4];
    rd(0, ra);
#pragma unroll
    for (int d = 0; d < ND; ++d) {
      v4s16 (&cur)[4] = (d & 1) ? rb : ra;
      v4s16 (&nxt)[4] = (d & 1) ? ra : rb;
      if (d < ND - 1) {
        rd(d + 1, nxt);
        asm volatile("s_waitcnt lgkmcnt(4)" : "+v"(cur[0]), "+v"(cur[1]), "+v"(cur[2]), "+v"(cur[3]));
      } else {
        asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(cur[0]), "+v"(cur[1]), "+v"(cur[2]), "+v"(cur[3]));
      }
      o[d] = mfma32b(frag(cur[0], cur[1]), pf[0], o[d]);
      o[d] = mfma32b(frag(cur[2], cur[3]), pf[1], o[d]);
    }
  };

  issue(0, page_of(pp0));
  if (n_pairs - pp0 > 1) issue(1, page_of(pp0 + 1));
  int nxt = page_of(pp0 + 2);
  int buf = 0;
  for (int pp = pp0; pp < n_pairs; ++pp) {
    if (pp + 1 < n_pairs) wait_vmcnt<OPS>(); else wait_vmcnt<0>();
    raw_barrier();  // pair pp visible to every wave; the slot consumed one step ago is free
    if (pp + 2 < n_pairs) {
      const int to = buf == 0 ? 2 : buf - 1;
      issue(to, nxt);
      nxt = page_of(pp + 3);
    }
    if (wave_live && pp * 32 <= wave_max && pp * 32 + 31 >= wave_low) {
      bf16x8 pf[2];
      const uint32_t so = buf * STAGE;
      softmax(qk(so), pp, pf);
      pv(so, pf);
    }
    buf = buf == 2 ? 0 : buf + 1;
  }

  {
    const auto sw = __builtin_amdgcn_permlane32_swap(__float_as_uint(l), __float_as_uint(l), false, false);
    l = __uint_as_float(sw[0]) + __uint_as_float(sw[1]);
  }
  if (!q_ok) return;
  float f = 1.f;
  if (a.sink) {
    const float m2 = m * a.scale_log2, s2 = a.sink[head] * kLog2e, M = fmaxf(m2, s2);
    f = exp2f(m2 - M);
    l = l * f + exp2f(s2 - M);
  }
  const float inv = l > 0.f ? f * gate_of(a, qs + qi, head) / l : 0.f;
  // O^T element e of dim block d is dim 32 d + 8 (e >> 2) + 4 h + (e & 3) of this lane's row
  uint16_t* orow = reinterpret_cast<uint16_t*>(a.out) + (size_t)(qs + qi) * a.out_row + head * a.V;
  const bool v4 = a.V % 4 == 0, gv = a.gate && a.gate_elem && a.gate_vec;
  // the gates of all elements are fetched together, ahead of the stores
  u32x2 z[ND][4];
  if (gv) {
    const uint16_t* g = reinterpret_cast<const uint16_t*>(a.gate) + (size_t)(qs + qi) * a.gate_stride + head * a.V;
#pragma unroll
    for (int d = 0; d < ND; ++d)
#pragma unroll
      for (int b = 0; b < 4; ++b) {
        const int c = 32 * d + 8 * b + 4 * h;
        z[d][b] = *reinterpret_cast<const u32x2*>(g + (c < a.V ? c : 0));
      }
  }
#pragma unroll
  for (int d = 0; d < ND; ++d)
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      const int c = 32 * d + 8 * b + 4 * h;
      float v[4] = {o[d][4 * b] * inv, o[d][4 * b + 1] * inv, o[d][4 * b + 2] * inv, o[d][4 * b + 3] * inv};
      if (gv) {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          v[j] *= __builtin_amdgcn_rcpf(1.f + __expf(-(j & 1 ? hi_bf(z[d][b][j >> 1]) : lo_bf(z[d][b][j >> 1]))));
      } else {
        gate_elems(a, qs + qi, head, c, v);
      }
      if (v4) {
        if (c < a.V) stn<4>(orow + c, v);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (c + j < a.V) orow[c + j] = f2bf(v[j]);
      }
    }
}

// Plain form: one wave per (query token, head), 64 keys at a time (a key per lane for the scores,
// a value element per lane for the output).  fp32 operands, or head sizes past the MFMA kernels.
template <typename E>
__global__ void __launch_bounds__(256) attn_any_kernel(AttnHdArgs a, const int* __restrict__ tile_seq,
                                                       const int* __restrict__ tile_q0, int tile_tokens) {
  extern __shared__ float sm_q[];  // [4][D]
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int tile = blockIdx.x, head = blockIdx.y, kvh = head / (a.H / a.G);
  const int s = tile_seq[tile];
  const int sub = blockIdx.z * 4 + wid;
  const int qi = tile_q0[tile] + sub;
  const int ql = a.q_len[s], ctx = a.ctx_len[s];
  if (sub >= tile_tokens || qi >= ql) return;  // whole waves; no barrier below
  const int tok = a.q_start[s] + qi, n_keys = max(0, ctx - ql + qi + 1), orow = a.by_tile ? tile : tok;
  const int k_lo = a.window > 0 ? max(0, n_keys - a.window) : 0;
  const E* kc = reinterpret_cast<const E*>(a.k_cache);
  const E* vc = reinterpret_cast<const E*>(a.v_cache);
  const E* q = reinterpret_cast<const E*>(a.q) + (size_t)orow * a.q_row + head * a.q_head;
  float* qs = sm_q + wid * a.D;
  const float* cs = a.rot ? a.rot + (size_t)min(max(n_keys - 1, 0), a.n_pos - 1) * a.n_rot : nullptr;
  for (int d = lane; d < a.D; d += 64) {
    const int r = d - a.rot_lo;
    float v = ld1(q + d);
    if (a.rot && r >= 0 && r < a.n_rot) {
      const float co = cs[r >> 1], si = cs[(a.n_rot >> 1) + (r >> 1)];
      v = r & 1 ? v * co + ld1(q + d - 1) * si : v * co - ld1(q + d + 1) * si;
    }
    qs[d] = v;
  }
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "workgroup");
  __builtin_amdgcn_wave_barrier();
  const int* bt = a.bt + (size_t)s * a.bt_stride;
  float acc[kHdMaxV / 64];
#pragma unroll
  for (int i = 0; i < kHdMaxV / 64; ++i) acc[i] = 0.f;
  float m = kLow, l = 0.f;
  for (int k0 = k_lo; k0 < n_keys; k0 += 64) {
    const int key = min(k0 + lane, n_keys - 1), n = min(64, n_keys - k0);
    const int line = a.xbase ? a.xbase[s] + key : min(max(bt[key / kPg], 0), a.num_blocks - 1) * kPg + key % kPg;
    const E* kr = kc + line / kPg * (kPg * a.k_pitch) + line % kPg * a.k_row + kvh * a.k_head;
    float dot = 0.f;
    for (int d = 0; d < a.D; ++d) dot = fmaf(qs[d], ld1(kr + d), dot);
    const float sc = lane < n ? dot * a.scale_log2 : -INFINITY;
    const float m_new = fmaxf(m, wave_max(sc)), alpha = exp2f(m - m_new);
    const float p = exp2f(sc - m_new);
    m = m_new;
    l = l * alpha + wave_sum(p);
#pragma unroll
    for (int i = 0; i < kHdMaxV / 64; ++i) acc[i] *= alpha;
    for (int j = 0; j < n; ++j) {
      const float pj = __shfl(p, j);
      const int lj = __shfl(line, j);
      const E* vr = vc + lj / kPg * (kPg * a.v_pitch) + lj % kPg * a.v_row + kvh * a.v_head;
#pragma unroll
      for (int i = 0; i < kHdMaxV / 64; ++i)
        if (i * 64 + lane < a.V) acc[i] = fmaf(pj, ld1(vr + i * 64 + lane), acc[i]);
    }
  }
  float f = 1.f;
  if (a.sink) {
    const float s2 = a.sink[head] * kLog2e, M = fmaxf(m, s2);
    f = exp2f(m - M);
    l = l * f + exp2f(s2 - M);
  }
  float inv = l > 0.f ? f / l : 0.f;
  const E* gate = reinterpret_cast<const E*>(a.gate) + (size_t)tok * a.gate_stride;
  if (a.gate && !a.gate_elem) inv /= 1.f + expf(-ld1(gate + head));
  E* dst = reinterpret_cast<E*>(a.out) + (size_t)orow * a.out_row + head * a.V;
#pragma unroll
  for (int i = 0; i < kHdMaxV / 64; ++i) {
    const int c = i * 64 + lane;
    if (c < a.V) st1(dst + c, a.gate && a.gate_elem ? acc[i] * inv / (1.f + expf(-ld1(gate + head * a.V + c))) : acc[i] * inv);
  }
}

template <typename E>
static void run_any(const AttnHdArgs& a, const int* tile_seq, const int* tile_q0, int num_tiles, int tile_tokens,
                    hipStream_t st) {
  attn_any_kernel<E><<<dim3(num_tiles, a.H, cdiv(tile_tokens, 4)), 256, (size_t)4 * a.D * 4, st>>>(a, tile_seq, tile_q0,
                                                                                               tile_tokens);
}

#define MLOP_HD_V(NKB, RUN)         \
  switch (a.VP / 64) {              \
    case 1: RUN(NKB, 1); break;     \
    case 2: RUN(NKB, 2); break;     \
    case 3: RUN(NKB, 3); break;     \
    default: RUN(NKB, 4); break;    \
  }
#define MLOP_HD(RUN)                          \
  switch (a.KP / 64) {                        \
    case 1: MLOP_HD_V(1, RUN) break;          \
    case 2: MLOP_HD_V(2, RUN) break;          \
    case 3: MLOP_HD_V(3, RUN) break;          \
    default: MLOP_HD_V(4, RUN) break;         \
  }

void launch_paged_hd(const AttnHdArgs& a, bool f32, float* part_o, float* part_ml, int* sem, const int* tile_seq,
                     const int* tile_q0, int num_tiles, int part_tokens, int nparts, hipStream_t st) {
  if (num_tiles == 0) return;
  if (f32) return run_any<float>(a, tile_seq, tile_q0, num_tiles, 1, st);
  if (latent_decode_ok(a, f32)) {
    launch_latent_decode(a, part_o, part_ml, tile_seq, tile_q0, num_tiles, part_tokens, nparts, st);
    return;
  }
  if (a.KP > kHdMaxDim || a.VP > kHdMaxDim) return run_any<uint16_t>(a, tile_seq, tile_q0, num_tiles, 1, st);
  const dim3 grid(num_tiles, a.G * cdiv(a.H / a.G, 16), nparts);
#define MLOP_RUN(K, V) \
  paged_hd_kernel<K, V><<<grid, 256, 0, st>>>(a, part_o, part_ml, sem, tile_seq, tile_q0, part_tokens, nparts)
  MLOP_HD(MLOP_RUN)
#undef MLOP_RUN
}

void launch_flash_hd(const AttnHdArgs& a, bool f32, const int* tile_seq, const int* tile_q0, int num_tiles,
                     hipStream_t st) {
  if (num_tiles == 0) return;
  if (f32) return run_any<float>(a, tile_seq, tile_q0, num_tiles, kHdTile, st);
  if (a.KP > kHdMaxDim || a.VP > kHdMaxDim) return run_any<uint16_t>(a, tile_seq, tile_q0, num_tiles, kHdTile, st);
#define MLOP_RUN(K, V) flash_hd_kernel<K, V><<<num_tiles * a.H, 256, 0, st>>>(a, tile_seq, tile_q0)
  MLOP_HD(MLOP_RUN)
#undef MLOP_RUN
}

}  // namespace mlop
