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

// Register form (head size a multiple of 8): a thread keeps its NQ q vectors and NK k vectors of 8
// elements from the sums of squares to the stores, with their norm weights, for TB tokens in turn
// (one norm-weight read per workgroup; the next token's row is fetched under this one's stores).
template <typename E, int NQ, int NK>
__global__ void __launch_bounds__(256) qk_norm_reg_kernel(QkNormArgs a, int TB) {
  __shared__ float scratch[2][4];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int nq = a.H * a.D, nk = a.G * a.D, nv = a.G * a.V, half = a.R / 2;
  int qc[NQ], qd[NQ], qdst[NQ], kc_[NK], kd[NK], kdst[NK];
  float qw[NQ][8], kw[NK][8];
#pragma unroll
  for (int i = 0; i < NQ; ++i) {
    const int c = (tid + 256 * i) * 8, h = c / a.D;
    qc[i] = c < nq ? c : -1;
    qd[i] = c - h * a.D;
    qdst[i] = h * a.KP + qd[i];
#pragma unroll
    for (int e = 0; e < 8; ++e) qw[i][e] = 1.f;
    if (a.q_w && c < nq) ldn<8>(a.q_w + c, qw[i]);
  }
#pragma unroll
  for (int i = 0; i < NK; ++i) {
    const int c = (tid + 256 * i) * 8, g = c / a.D;
    kc_[i] = c < nk ? c : -1;
    kd[i] = c - g * a.D;
    kdst[i] = g * a.BS * a.KP + kd[i];
#pragma unroll
    for (int e = 0; e < 8; ++e) kw[i][e] = 1.f;
    if (a.k_w && c < nk) ldn<8>(a.k_w + c, kw[i]);
  }
  const float lam = a.v_first ? *a.lam : 0.f;
  const bool v8 = a.V % 8 == 0 && a.ldf % 8 == 0 && (reinterpret_cast<uintptr_t>(a.v_first) & 15) == 0;
  const bool r8 = a.R % 8 == 0;  // whole vectors turn, or none of their pairs does
  const int pad = a.KP - a.D;
  const int t_end = min(a.T, ((int)blockIdx.x + 1) * TB);
  for (int t = blockIdx.x * TB; t < t_end; ++t) {
    const E* row = reinterpret_cast<const E*>(a.proj) + (size_t)t * a.ldp;
    float q[NQ][8], k[NK][8], sq = 0.f, sk = 0.f;
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
#pragma unroll
      for (int e = 0; e < 8; ++e) q[i][e] = 0.f;
      if (qc[i] >= 0) ldn<8>(row + qc[i], q[i]);
    }
#pragma unroll
    for (int i = 0; i < NK; ++i) {
#pragma unroll
      for (int e = 0; e < 8; ++e) k[i][e] = 0.f;
      if (kc_[i] >= 0) ldn<8>(row + nq + kc_[i], k[i]);
    }
    const float* cs = a.cos_sin + (size_t)a.pos[t] * a.R;
    const int slot = a.slots[t];
    float iq = 1.f, ik = 1.f;
    if (a.q_w) {
#pragma unroll
      for (int i = 0; i < NQ; ++i)
#pragma unroll
        for (int e = 0; e < 8; ++e) sq = fmaf(q[i][e], q[i][e], sq);
#pragma unroll
      for (int i = 0; i < NK; ++i)
#pragma unroll
        for (int e = 0; e < 8; ++e) sk = fmaf(k[i][e], k[i][e], sk);
      sq = wave_sum(sq);
      sk = wave_sum(sk);
      if (lane == 0) scratch[0][wid] = sq, scratch[1][wid] = sk;
      __syncthreads();
      sq = scratch[0][0] + scratch[0][1] + scratch[0][2] + scratch[0][3];
      sk = scratch[1][0] + scratch[1][1] + scratch[1][2] + scratch[1][3];
      __syncthreads();
      iq = 1.f / sqrtf(sq / (float)nq + a.eps);
      ik = 1.f / sqrtf(sk / (float)nk + a.eps);
    }
    auto turn = [&](float (&o)[8], const float (&w)[8], float inv, int d) {
#pragma unroll
      for (int e = 0; e < 8; ++e) o[e] *= inv * w[e];
      if (r8) {
        if (d < a.R) {
          float c[4], s[4];
          ldn<4>(cs + (d >> 1), c);
          ldn<4>(cs + half + (d >> 1), s);
#pragma unroll
          for (int e = 0; e < 8; e += 2) {
            const float x = o[e], y = o[e + 1];
            o[e] = x * c[e >> 1] - y * s[e >> 1];
            o[e + 1] = y * c[e >> 1] + x * s[e >> 1];
          }
        }
        return;
      }
#pragma unroll
      for (int e = 0; e < 8; e += 2) {
        if (d + e < a.R) {
          const float c = cs[(d + e) >> 1], s = cs[half + ((d + e) >> 1)];
          const float x = o[e], y = o[e + 1];
          o[e] = x * c - y * s;
          o[e + 1] = y * c + x * s;
        }
      }
    };
    E* qo = reinterpret_cast<E*>(a.q_out) + (size_t)t * a.H * a.KP;
#pragma unroll
    for (int i = 0; i < NQ; ++i)
      if (qc[i] >= 0) {
        turn(q[i], qw[i], iq, qd[i]);
        stn<8>(qo + qdst[i], q[i]);
      }
    if (pad)
      for (int c = tid; c < a.H * pad; c += 256) st1(qo + (size_t)(c / pad) * a.KP + a.D + c % pad, 0.f);
    if (slot < 0) continue;
    const int blk = slot / a.BS, off = slot - blk * a.BS;
    E* ko = reinterpret_cast<E*>(a.k_cache) + ((size_t)blk * a.G * a.BS + off) * a.KP;
#pragma unroll
    for (int i = 0; i < NK; ++i)
      if (kc_[i] >= 0) {
        turn(k[i], kw[i], ik, kd[i]);
        stn<8>(ko + kdst[i], k[i]);
      }
    E* vo = reinterpret_cast<E*>(a.v_cache) + ((size_t)blk * a.G * a.BS + off) * a.VP;
    const E* v0 = row + nq + nk;
    const E* vf = reinterpret_cast<const E*>(a.v_first) + (a.v_first ? (size_t)t * a.ldf : 0);
    if (v8) {
      for (int c = tid * 8; c < nv; c += 2048) {
        const int g = c / a.V, d = c - g * a.V;
        float v[8];
        ldn<8>(v0 + c, v);
        if (a.v_first) {
          float f[8];
          ldn<8>(vf + c, f);
#pragma unroll
          for (int e = 0; e < 8; ++e) v[e] = (1.f - lam) * v[e] + lam * f[e];
        }
        stn<8>(vo + (size_t)g * a.BS * a.VP + d, v);
      }
    } else {
      for (int c = tid; c < nv; c += 256) {
        const int g = c / a.V, d = c - g * a.V;
        float v = ld1(v0 + c);
        if (a.v_first) v = (1.f - lam) * v + lam * ld1(vf + c);
        st1(vo + (size_t)g * a.BS * a.VP + d, v);
      }
    }
  }
}

template <typename E>
static void run_qk(const QkNormArgs& a, hipStream_t st) {
  const int nq = cdiv(a.H * a.D, 2048), nk = cdiv(a.G * a.D, 2048);
  if (a.D % 8 == 0 && a.ldp % 8 == 0 && nq <= 4 && nk <= 2) {
    const int TB = a.T >= 4096 ? 4 : 1, grid = cdiv(a.T, TB);
    if (nk == 2) qk_norm_reg_kernel<E, 4, 2><<<grid, 256, 0, st>>>(a, TB);
    else if (nq <= 1) qk_norm_reg_kernel<E, 1, 1><<<grid, 256, 0, st>>>(a, TB);
    else if (nq <= 2) qk_norm_reg_kernel<E, 2, 1><<<grid, 256, 0, st>>>(a, TB);
    else qk_norm_reg_kernel<E, 4, 1><<<grid, 256, 0, st>>>(a, TB);
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
