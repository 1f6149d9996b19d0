// From the fused projection rows [q | k | v | ...] of a step to attention's operands:
//   * RMSNorm of all q rows at once and of all k rows at once (before the split into heads);
//   * rotary positions on the first R dims of every q / k head, dimension 2i paired with 2i + 1;
//   * v <- (1 - lam) v + lam v_first (value mixing with an earlier layer's values of the token);
//   * q to [T, H, KP] (dims past D zero), k and v straight into the paged cache.
// One workgroup per token; the projection row is read twice (the second time from cache).
#include "elem.h"
#include "hybrid.h"

namespace mlop {

template <typename E, int VEC>
__global__ void __launch_bounds__(256) qk_norm_kernel(QkNormArgs a) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, tid = threadIdx.x;
  const E* row = reinterpret_cast<const E*>(a.proj) + (size_t)t * a.ldp;
  const int nq = a.H * a.D, nk = a.G * a.D;
  float iq = 1.f, ik = 1.f;
  if (a.q_w) {
    float sq = 0.f, sk = 0.f, v[VEC];
    for (int c = tid * VEC; c < nq; c += 256 * VEC) {
      ldn<VEC>(row + c, v);
#pragma unroll
      for (int e = 0; e < VEC; ++e) sq = fmaf(v[e], v[e], sq);
    }
    for (int c = tid * VEC; c < nk; c += 256 * VEC) {
      ldn<VEC>(row + nq + c, v);
#pragma unroll
      for (int e = 0; e < VEC; ++e) sk = fmaf(v[e], v[e], sk);
    }
    sq = block_sum(sq, scratch);
    sk = block_sum(sk, scratch);
    iq = 1.f / sqrtf(sq / (float)nq + a.eps);
    ik = 1.f / sqrtf(sk / (float)nk + a.eps);
  }
  const float* cs = a.cos_sin + (size_t)a.pos[t] * a.R;
  const int half = a.R / 2;
  // VEC elements of head dim d.. of one head: normed, rotated
  auto turn = [&](const E* src, const float* w, float inv, int d, float (&o)[VEC]) {
    ldn<VEC>(src, o);
    if (w) {
      float wv[VEC];
      ldn<VEC>(w, wv);
#pragma unroll
      for (int e = 0; e < VEC; ++e) o[e] *= inv * wv[e];
    }
#pragma unroll
    for (int e = 0; e < VEC; e += 2) {
      if (d + e < a.R) {
        const float c = cs[(d + e) >> 1], s = cs[half + ((d + e) >> 1)];
        const float x = o[e], y = o[e + 1];
        o[e] = x * c - y * s;
        o[e + 1] = y * c + x * s;
      }
    }
  };
  E* q = reinterpret_cast<E*>(a.q_out) + (size_t)t * a.H * a.KP;
  for (int c = tid * VEC; c < nq; c += 256 * VEC) {
    const int h = c / a.D, d = c - h * a.D;
    float o[VEC];
    turn(row + c, a.q_w ? a.q_w + c : nullptr, iq, d, o);
    stn<VEC>(q + (size_t)h * a.KP + d, o);
  }
  const int pad = a.KP - a.D;
  for (int c = tid; c < a.H * pad; c += 256) st1(q + (size_t)(c / pad) * a.KP + a.D + c % pad, 0.f);
  const int slot = a.slots[t];
  if (slot < 0) return;
  const int blk = slot / a.BS, off = slot - blk * a.BS;
  E* kc = reinterpret_cast<E*>(a.k_cache) + ((size_t)blk * a.G * a.BS + off) * a.KP;
  for (int c = tid * VEC; c < nk; c += 256 * VEC) {
    const int g = c / a.D, d = c - g * a.D;
    float o[VEC];
    turn(row + nq + c, a.k_w ? a.k_w + c : nullptr, ik, d, o);
    stn<VEC>(kc + (size_t)g * a.BS * a.KP + d, o);
  }
  E* vc = reinterpret_cast<E*>(a.v_cache) + ((size_t)blk * a.G * a.BS + off) * a.VP;
  const E* v0 = row + nq + nk;
  const E* vf = reinterpret_cast<const E*>(a.v_first) + (a.v_first ? (size_t)t * a.ldf : 0);
  const float lam = a.v_first ? *a.lam : 0.f;
  for (int c = tid; c < a.G * a.V; c += 256) {
    const int g = c / a.V, d = c - g * a.V;
    float v = ld1(v0 + c);
    if (a.v_first) v = (1.f - lam) * v + lam * ld1(vf + c);
    st1(vc + (size_t)g * a.BS * a.VP + d, v);
  }
}

// Vector form (head sizes multiples of 8): the token's [q | k | v] vectors of 8 elements are dealt to
// the threads of one workgroup (NI each, one at the usual sizes), which keep them, and their norm
// weights, in registers from the sums of squares to the stores, for TB tokens in turn.
template <typename E, int NI>
__global__ void __launch_bounds__(1024) qk_norm_vec_kernel(QkNormArgs a, int TB) {
  __shared__ float scratch[2][2][16];
  const int tid = threadIdx.x, BT = blockDim.x, lane = tid & 63, wid = tid >> 6, NWv = BT >> 6;
  const int nq = a.H * a.D, nk = a.G * a.D, nv = a.G * a.V, half = a.R / 2;
  enum { NONE, Q, K, V };
  int kind[NI], d[NI], dst[NI];
  float w[NI][8];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = (tid + BT * i) * 8;
    kind[i] = c < nq ? Q : c < nq + nk ? K : c < nq + nk + nv ? V : NONE;
    const int cc = kind[i] == Q ? c : kind[i] == K ? c - nq : c - nq - nk;
    const int sz = kind[i] == V ? a.V : a.D, h = cc / sz;
    d[i] = kind[i] == V ? a.R : cc - h * sz;  // (values never turn)
    dst[i] = (kind[i] == Q ? h * a.KP : h * a.BS * (kind[i] == V ? a.VP : a.KP)) + cc - h * sz;
#pragma unroll
    for (int e = 0; e < 8; ++e) w[i][e] = 1.f;
    if (a.q_w && kind[i] == Q) ldn<8>(a.q_w + cc, w[i]);
    if (a.k_w && kind[i] == K) ldn<8>(a.k_w + cc, w[i]);
  }
  const float lam = a.v_first ? *a.lam : 0.f;
  const bool r8 = a.R > 0 && a.R % 8 == 0;  // whole vectors turn, or none of their pairs does
  const int pad = a.KP - a.D;
  const int t_end = min(a.T, ((int)blockIdx.x + 1) * TB);
  for (int t = blockIdx.x * TB; t < t_end; ++t) {
    const E* row = reinterpret_cast<const E*>(a.proj) + (size_t)t * a.ldp;
    float x[NI][8];
#pragma unroll
    for (int i = 0; i < NI; ++i) {
ldn<8>(row + (kind[i] == NONE ? 0 : (tid + BT * i) * 8), x[i]);
    }
    const float* cs = a.cos_sin + (size_t)a.pos[t] * a.R;
    const int slot = a.slots[t];
    // cos / sin and the values to mix in are fetched beside the row, unconditionally (clamped)
    float cc[NI][4], sc4[NI][4], f[NI][8];
    if (r8) {
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        const int o = d[i] < a.R ? d[i] >> 1 : 0;
        ldn<4>(cs + o, cc[i]);
        ldn<4>(cs + half + o, sc4[i]);
      }
    }
    if (a.v_first) {
#pragma unroll
      for (int i = 0; i < NI; ++i)
        ldn<8>(reinterpret_cast<const E*>(a.v_first) + (size_t)t * a.ldf + (kind[i] == V ? (tid + BT * i) * 8 - nq - nk : 0),
               f[i]);
    }
    float inv[2] = {1.f, 1.f};
    if (a.q_w) {
      float sq = 0.f, sk = 0.f;
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        float s = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) s = fmaf(x[i][e], x[i][e], s);
        sq += kind[i] == Q ? s : 0.f;
        sk += kind[i] == K ? s : 0.f;
      }
      sq = wave_sum(sq);
      sk = wave_sum(sk);
      // double-buffered over the tokens: one barrier each, for LDS only (stores stay in flight)
      float (*sc)[16] = scratch[t & 1];
      if (lane == 0) sc[0][wid] = sq, sc[1][wid] = sk;
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      raw_barrier();
      sq = sk = 0.f;
      for (int k = 0; k < NWv; ++k) sq += sc[0][k], sk += sc[1][k];
      inv[0] = 1.f / sqrtf(sq / (float)nq + a.eps);
      inv[1] = 1.f / sqrtf(sk / (float)nk + a.eps);
    }
    const int blk = slot >= 0 ? slot / a.BS : 0, off = slot - blk * a.BS;
    E* qo = reinterpret_cast<E*>(a.q_out) + (size_t)t * a.H * a.KP;
    E* ko = reinterpret_cast<E*>(a.k_cache) + ((size_t)blk * a.G * a.BS + off) * a.KP;
    E* vo = reinterpret_cast<E*>(a.v_cache) + ((size_t)blk * a.G * a.BS + off) * a.VP;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      if (kind[i] == NONE || (kind[i] != Q && slot < 0)) continue;
      if (kind[i] == V) {
        if (a.v_first) {
#pragma unroll
          for (int e = 0; e < 8; ++e) x[i][e] = (1.f - lam) * x[i][e] + lam * f[i][e];
        }
        stn<8>(vo + dst[i], x[i]);
        continue;
      }
      const float n = kind[i] == Q ? inv[0] : inv[1];
#pragma unroll
      for (int e = 0; e < 8; ++e) x[i][e] *= n * w[i][e];
      if (d[i] < a.R) {
        float c[4], s[4];
        if (r8) {
#pragma unroll
          for (int e = 0; e < 4; ++e) c[e] = cc[i][e], s[e] = sc4[i][e];
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const bool in = d[i] + 2 * e < a.R;
            c[e] = in ? cs[(d[i] >> 1) + e] : 1.f;
            s[e] = in ? cs[half + (d[i] >> 1) + e] : 0.f;
          }
        }
#pragma unroll
        for (int e = 0; e < 8; e += 2) {
          const float u = x[i][e], y = x[i][e + 1];
          x[i][e] = u * c[e >> 1] - y * s[e >> 1];
          x[i][e + 1] = y * c[e >> 1] + u * s[e >> 1];
        }
      }
      stn<8>((kind[i] == Q ? qo : ko) + dst[i], x[i]);
    }
    if (pad)
      for (int c = tid; c < a.H * pad; c += BT) st1(qo + (size_t)(c / pad) * a.KP + a.D + c % pad, 0.f);
  }
}

template <typename E>
static void run_qk(const QkNormArgs& a, hipStream_t st) {
  const int items = cdiv(a.H * a.D + a.G * (a.D + a.V), 8);
  const bool vf = !a.v_first || (a.ldf % 8 == 0 && (reinterpret_cast<uintptr_t>(a.v_first) & 15) == 0);
  if (a.D % 8 == 0 && a.V % 8 == 0 && a.ldp % 8 == 0 && vf && items <= 4096) {
    const int ni = items <= 1024 ? 1 : items <= 2048 ? 2 : 4;
    const int block = cdiv(cdiv(items, ni), 64) * 64, TB = a.T >= 8192 ? 8 : a.T >= 2048 ? 4 : 1, grid = cdiv(a.T, TB);
    if (ni == 1) qk_norm_vec_kernel<E, 1><<<grid, block, 0, st>>>(a, TB);
    else if (ni == 2) qk_norm_vec_kernel<E, 2><<<grid, block, 0, st>>>(a, TB);
    else qk_norm_vec_kernel<E, 4><<<grid, block, 0, st>>>(a, TB);
  } else if (a.D % 8 == 0 && a.ldp % 8 == 0) {
    qk_norm_kernel<E, 8><<<a.T, 256, 0, st>>>(a);
  } else {
    qk_norm_kernel<E, 2><<<a.T, 256, 0, st>>>(a);
  }
}

void launch_qk_norm(const QkNormArgs& a, bool f32, hipStream_t st) {
  if (a.T == 0) return;
  if (f32) run_qk<float>(a, st);
  else run_qk<uint16_t>(a, st);
}

// Per-head form: every query and key head divided by its own root mean square, one weight for all of them; the
// values are columns of their own or the keys as given.  Vector kernel: LPH lanes of a wave hold a head's 8-element
// vectors in registers from the sum of squares to the stores, HPT heads of one token in turn (fetched together).
template <typename E, int LPH, int HPT>
__global__ void __launch_bounds__(256) qk_head_norm_vec_kernel(QkHeadNormArgs a) {
  const int units = cdiv(a.H + a.G, HPT), c = threadIdx.x % LPH * 8;
  const long unit = (long)blockIdx.x * (256 / LPH) + threadIdx.x / LPH;
  if (unit >= (long)a.T * units) return;  // whole groups of lanes; no barrier below
  const int t = (int)(unit / units), h0 = (int)(unit % units) * HPT;
  const bool in = c < a.D;
  const E* qr = reinterpret_cast<const E*>(a.q) + (size_t)t * a.ldq;
  const E* kr = reinterpret_cast<const E*>(a.k) + (size_t)t * a.ldk;
  float x[HPT][8];
#pragma unroll
  for (int i = 0; i < HPT; ++i) {
    const int h = min(h0 + i, a.H + a.G - 1);
    ldn<8>((h < a.H ? qr + h * a.D : kr + (h - a.H) * a.D) + (in ? c : 0), x[i]);
  }
  // the weights, cos and sin fetched beside the heads, unconditionally (clamped)
  float qw[8], kw[8], co[4], si[4];
  ldn<8>(a.q_w + (in ? c : 0), qw);
  ldn<8>(a.k_w + (in ? c : 0), kw);
  const int half = a.R >> 1;
  const float* cs = a.cos_sin + (size_t)a.pos[t] * a.R;
  if (a.R % 8 == 0) {
    const int o = c < a.R ? c >> 1 : 0;
    if (a.R) {
      ldn<4>(cs + o, co);
      ldn<4>(cs + half + o, si);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) co[e] = c < a.R ? co[e] : 1.f, si[e] = c < a.R ? si[e] : 0.f;
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const bool r = c + 2 * e < a.R;
      co[e] = r ? cs[(c >> 1) + e] : 1.f;
      si[e] = r ? cs[half + (c >> 1) + e] : 0.f;
    }
  }
  const int slot = a.slots[t], blk = slot >= 0 ? slot / a.BS : 0, off = slot - blk * a.BS;
#pragma unroll
  for (int i = 0; i < HPT; ++i) {
    const int h = h0 + i, g = h - a.H;
    float s = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) s = fmaf(x[i][e], x[i][e], s);
    s = in ? s : 0.f;
    s += detail::dpp<0xB1>(s);
    s += detail::dpp<0x4E>(s);
    s += detail::dpp<0x141>(s);  // 8 lanes
    if constexpr (LPH >= 16) s += detail::dpp<0x140>(s);
    if constexpr (LPH >= 32) s += __shfl_xor(s, 16);
    if constexpr (LPH >= 64) s += __shfl_xor(s, 32);
    if (h >= a.H + a.G || (g >= 0 && slot < 0)) continue;
    const float inv = 1.f / sqrtf(s / (float)a.D + a.eps);
    float o[8];
#pragma unroll
    for (int e = 0; e < 8; e += 2) {
      const float u = x[i][e] * inv * (g < 0 ? qw[e] : kw[e]), y = x[i][e + 1] * inv * (g < 0 ? qw[e + 1] : kw[e + 1]);
      o[e] = u * co[e >> 1] - y * si[e >> 1];
      o[e + 1] = y * co[e >> 1] + u * si[e >> 1];
    }
    if (g < 0) {
#pragma unroll
      for (int e = 0; e < 8; ++e) o[e] = in ? o[e] : 0.f;
      if (c < a.KP) stn<8>(reinterpret_cast<E*>(a.q_out) + ((size_t)t * a.H + h) * a.KP + c, o);
      continue;
    }
    const size_t line = ((size_t)blk * a.G + g) * a.BS + off;
    if (in) stn<8>(reinterpret_cast<E*>(a.k_cache) + line * a.KP + c, o);
    E* vo = reinterpret_cast<E*>(a.v_cache) + line * a.VP;
    if (!a.v) {
      if (in) stn<8>(vo + c, x[i]);
    } else {
      const E* vr = reinterpret_cast<const E*>(a.v) + (size_t)t * a.ldv + (size_t)g * a.V;
      for (int e = threadIdx.x % LPH; e < a.V; e += LPH) st1(vo + e, ld1(vr + e));
    }
  }
}

// any head size and alignment: a wave per (token, head)
template <typename E>
__global__ void __launch_bounds__(256) qk_head_norm_any_kernel(QkHeadNormArgs a) {
  const int lane = threadIdx.x & 63;
  const long unit = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (unit >= (long)a.T * (a.H + a.G)) return;
  const int t = (int)(unit / (a.H + a.G)), h = (int)(unit % (a.H + a.G)), g = h - a.H;
  const E* src = g < 0 ? reinterpret_cast<const E*>(a.q) + (size_t)t * a.ldq + (size_t)h * a.D
                       : reinterpret_cast<const E*>(a.k) + (size_t)t * a.ldk + (size_t)g * a.D;
  float s = 0.f;
  for (int d = lane; d < a.D; d += 64) {
    const float x = ld1(src + d);
    s = fmaf(x, x, s);
  }
  const float inv = 1.f / sqrtf(wave_sum(s) / (float)a.D + a.eps);
  const float* w = g < 0 ? a.q_w : a.k_w;
  const float* cs = a.cos_sin + (size_t)a.pos[t] * a.R;
  auto turned = [&](int d) {
    const float x = ld1(src + d) * inv * w[d];
    if (d >= a.R) return x;
    const float y = ld1(src + (d ^ 1)) * inv * w[d ^ 1], co = cs[d >> 1], si = cs[(a.R >> 1) + (d >> 1)];
    return d & 1 ? x * co + y * si : x * co - y * si;
  };
  if (g < 0) {
    E* q = reinterpret_cast<E*>(a.q_out) + ((size_t)t * a.H + h) * a.KP;
    for (int d = lane; d < a.KP; d += 64) st1(q + d, d < a.D ? turned(d) : 0.f);
    return;
  }
  const int slot = a.slots[t];
  if (slot < 0) return;
  const size_t line = ((size_t)(slot / a.BS) * a.G + g) * a.BS + slot % a.BS;
  E* ko = reinterpret_cast<E*>(a.k_cache) + line * a.KP;
  E* vo = reinterpret_cast<E*>(a.v_cache) + line * a.VP;
  for (int d = lane; d < a.D; d += 64) st1(ko + d, turned(d));
  const E* vr = a.v ? reinterpret_cast<const E*>(a.v) + (size_t)t * a.ldv + (size_t)g * a.V : src;
  for (int d = lane; d < a.V; d += 64) st1(vo + d, ld1(vr + d));
}

template <typename E>
static void run_qk_head(const QkHeadNormArgs& a, hipStream_t st) {
  const bool al = ((reinterpret_cast<uintptr_t>(a.q) | reinterpret_cast<uintptr_t>(a.k)) & 15) == 0;
  if (al && a.D % 8 == 0 && a.ldq % 8 == 0 && a.ldk % 8 == 0 && a.KP <= 512 && a.VP % 8 == 0) {
    const int HPT = a.T >= 1024 ? 4 : 1;
#define MLOP_QKH_N(LPH, N) \
  qk_head_norm_vec_kernel<E, LPH, N><<<(int)(((long)a.T * cdiv(a.H + a.G, N) * LPH + 255) / 256), 256, 0, st>>>(a)
#define MLOP_QKH(LPH) \
  if (HPT == 4) MLOP_QKH_N(LPH, 4); else MLOP_QKH_N(LPH, 1)
    if (a.KP <= 64) { MLOP_QKH(8); }
    else if (a.KP <= 128) { MLOP_QKH(16); }
    else if (a.KP <= 256) { MLOP_QKH(32); }
    else { MLOP_QKH(64); }
#undef MLOP_QKH
#undef MLOP_QKH_N
  } else {
    qk_head_norm_any_kernel<E><<<(int)(((long)a.T * (a.H + a.G) + 3) / 4), 256, 0, st>>>(a);
  }
}

void launch_qk_head_norm(const QkHeadNormArgs& a, bool f32, hipStream_t st) {
  if (a.T == 0) return;
  if (f32) run_qk_head<float>(a, st);
  else run_qk_head<uint16_t>(a, st);
}

}  // namespace mlop
