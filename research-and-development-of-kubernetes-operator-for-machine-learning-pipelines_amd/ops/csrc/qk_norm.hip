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

void launch_qk_norm(const QkNormArgs& a, bool f32, hipStream_t st) {
  if (a.T == 0) return;
  const bool v8 = a.D % 8 == 0 && a.ldp % 8 == 0;
  if (f32) {
    if (v8) qk_norm_kernel<float, 8><<<a.T, 256, 0, st>>>(a);
    else qk_norm_kernel<float, 2><<<a.T, 256, 0, st>>>(a);
  } else {
    if (v8) qk_norm_kernel<uint16_t, 8><<<a.T, 256, 0, st>>>(a);
    else qk_norm_kernel<uint16_t, 2><<<a.T, 256, 0, st>>>(a);
  }
}

}  // namespace mlop
