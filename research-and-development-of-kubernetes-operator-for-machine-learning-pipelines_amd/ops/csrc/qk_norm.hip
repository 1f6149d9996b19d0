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

}  // namespace mlop
