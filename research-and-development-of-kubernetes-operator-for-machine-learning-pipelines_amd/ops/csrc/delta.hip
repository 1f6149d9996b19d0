// Generalized delta rule: per head a matrix state S [dk, dv] in fp32 with a decay per key channel and a
// rank-one removal,
//
//   S_t = diag(w_t) S_{t-1} - (a_t u_t) (u_t^T S_{t-1}) + k_t v_t^T,      o_t = S_t^T r_t
//   u = k / sqrt(sum(k^2) + unit_eps),  log w = -decay_scale sigmoid(W2 tanh(w1) + w0),  a = sigmoid(a + a_b)
//
// Everything of the recurrence is fp32 (the projections arrive in the model dtype); the matrix products
// use the fp32 MFMA.  Three kernels:
//
//   delta_rows_kernel    one-token rows: a workgroup per (row, head) reads the state once for u^T S and
//                        (w r)^T S together, keeps it in registers and writes the new one (HBM-bound);
//   delta_block_kernel   blocks of 16 prompt tokens, all in parallel: with b_t the running sum of log w
//                        in a block and x_t = S_{t-1}^T u_t, the recurrence is linear in the block's start:
//                          X = W S + M V                       W = (I - T)^-1 B~, M = (I - T)^-1 (B~ K~^T)_<
//                          O = R S + A V                       R = R~ + (R~ A~^T)_<= W, A = (R~ K~^T)_<= + (R~ A~^T)_<= M
//                          S <- diag(e^{b_16}) S + K^ V + A^ X
//                        B~_t = u_t e^{b_{t-1}},  R~_t = r_t e^{b_t},  K~_j = k_j e^{-b_j},  A~_j = -(a_j u_j) e^{-b_j},
//                        T = (B~ A~^T)_<,  K^_j = k_j e^{b_16 - b_j},  A^_j = -(a_j u_j) e^{b_16 - b_j}.
//                        decay_scale bounds e^{-b_j}, so the factors stay in range;
//   delta_walk_kernel    a workgroup per (sequence, head, 16 columns of dv) walks a portion's blocks with
//                        the state in its accumulators, its 4 waves splitting dk; one barrier per block.
//
// A sequence's first token starts from the zero state whatever its slot holds.
#include <algorithm>

#include "mixers.h"
#include "recur.h"

namespace mlop {

namespace {

constexpr int kBlk = 16;
constexpr int kDeltaMaxDk = 256;
constexpr float kMaxBlockDecay = 60.f;  // |b_16| the factored form allows (natural log)

// per (block, head) in the workspace: W, R [16][dkp] | K^, A^ [dkp][16] | e^{b_16} [dkp] | M, A [16][16]
__host__ __device__ constexpr int delta_dkp(int dk) { return (dk + 15) / 16 * 16; }
__host__ __device__ constexpr long delta_per(int dkp) { return (long)dkp * 65 + 512; }

// log2 decay of a channel from its logit
__device__ __forceinline__ float log2_decay(const DeltaArgs& a, float z) { return -a.decay_scale * kLog2E * sigmoid_hw(z); }

}  // namespace

// NR: key rows of a strip that a thread keeps in registers from their loads, in front of everything else,
// to the stores (one strip per thread, then); 0: the state is read twice.
template <typename E, int VEC, int BT, int NR, bool NT>
__global__ void __launch_bounds__(BT) delta_rows_kernel(DeltaArgs a, StepRows r, const int* __restrict__ rows) {
  extern __shared__ float sm[];
  __shared__ float scratch[3][BT / 64];
  const int s = rows[blockIdx.x], h = blockIdx.y, tid = threadIdx.x;
  const int dk = a.dk, dv = a.dv, HK = a.H * dk, HV = a.H * dv;
  float* w1 = sm;                  // [rank]
  float* wv = w1 + a.rank;         // [dk] each: decay, unit key, removal, key, w r
  float* uv = wv + dk;
  float* au = uv + dk;
  float* kv = au + dk;
  float* rv = kv + dk;
  float* red = rv + dk;            // [2][BT * VEC]
  float* zc = red + 2 * BT * VEC;  // [BT * VEC]
  const int ql = r.q_len[s], ctx = r.ctx_len[s], q0 = r.q_start[s];
  E* op = reinterpret_cast<E*>(a.o) + (size_t)q0 * HV + h * dv;
  if (ctx < ql || s >= r.n_slots) {  // graph padding: holds no state
    for (int t = 0; t < ql; ++t)
      for (int c = tid; c < dv; c += BT) st1(op + (size_t)t * HV + c, 0.f);
    return;
  }
  float* S = a.state + ((size_t)s * a.H + h) * dk * dv;
  const int nstrip = dv / VEC, per = min(nstrip, BT), RG = BT / per, rg = tid / per;
  for (int t = 0; t < ql; ++t) {
    const E* row = reinterpret_cast<const E*>(a.proj) + (size_t)(q0 + t) * a.ldp;
    const bool fresh = ctx - ql + t == 0;
    float x[NR ? NR : 1][VEC];
    auto get = [&](int strip, int d, float (&v)[VEC]) {
      if (fresh) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] = 0.f;
      } else {
        ld_state<NT>(S + strip * VEC + (size_t)d * dv, v);
      }
    };
    if constexpr (NR > 0) {
      if (rg < RG) {
#pragma unroll
        for (int i = 0; i < NR; ++i)
          if (rg + i * RG < dk) get(tid % per, rg + i * RG, x[i]);
      }
    }
    for (int i = tid; i < a.rank; i += BT) w1[i] = tanh_hw(ld1(row + 3 * HK + HV + i));
    __syncthreads();
    float ss = 0.f, rk = 0.f, ra = 0.f;
    for (int d = tid; d < dk; d += BT) {
      const int n = h * dk + d;
      const float k = ld1(row + HK + n), rr = ld1(row + n);
      const float al = sigmoid_hw(ld1(row + 2 * HK + HV + n) + a.a_b[n]);
      float z = a.w0[n];
      const E* w2 = reinterpret_cast<const E*>(a.w2) + (size_t)n * a.rank;
      if (a.rank % 8 == 0) {
        for (int i = 0; i < a.rank; i += 8) {
          float wr[8];
          ldn<8>(w2 + i, wr);
#pragma unroll
          for (int e = 0; e < 8; ++e) z = fmaf(wr[e], w1[i + e], z);
        }
      } else {
        for (int i = 0; i < a.rank; ++i) z = fmaf(ld1(w2 + i), w1[i], z);
      }
      const float w = exp2_f(log2_decay(a, z));
      wv[d] = w;
      kv[d] = k;
      rv[d] = rr * w;
      au[d] = al;
      ss = fmaf(k, k, ss);
      rk = fmaf(rr, k, rk);
      ra = fmaf(rr, al * k, ra);
    }
    ss = wave_sum(ss);
    rk = wave_sum(rk);
    ra = wave_sum(ra);
    if ((tid & 63) == 0) {
      scratch[0][tid >> 6] = ss;
      scratch[1][tid >> 6] = rk;
      scratch[2][tid >> 6] = ra;
    }
    __syncthreads();
    ss = rk = ra = 0.f;
#pragma unroll
    for (int w = 0; w < BT / 64; ++w) {
      ss += scratch[0][w];
      rk += scratch[1][w];
      ra += scratch[2][w];
    }
    const float inv = 1.f / sqrtf(ss + a.unit_eps);
    ra *= inv;  // r . (a u)
    for (int d = tid; d < dk; d += BT) {
      const float u = kv[d] * inv;
      uv[d] = u;
      au[d] *= u;
    }
    __syncthreads();
    for (int s0 = 0; s0 < nstrip; s0 += per) {
      const int strip = s0 + tid % per;
      const bool on = rg < RG && strip < nstrip;
      float z[VEC], y[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) z[e] = y[e] = 0.f;
      auto sums = [&](int d, const float (&v)[VEC]) {
        const float u = uv[d], rw = rv[d];
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
          z[e] = fmaf(u, v[e], z[e]);
          y[e] = fmaf(rw, v[e], y[e]);
        }
      };
      if (on) {
        if constexpr (NR > 0) {
#pragma unroll
          for (int i = 0; i < NR; ++i)
            if (rg + i * RG < dk) sums(rg + i * RG, x[i]);
        } else {
          for (int d = rg; d < dk; d += RG) {
            get(strip, d, x[0]);
            sums(d, x[0]);
          }
        }
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        red[tid * VEC + e] = z[e];
        red[(BT + tid) * VEC + e] = y[e];
      }
      __syncthreads();
      for (int c = tid; c < per * VEC; c += BT) {
        const int cc = s0 * VEC + c;
        if (cc < dv) {
          float zz = 0.f, yy = 0.f;
          for (int g = 0; g < RG; ++g) {
            zz += red[g * per * VEC + c];
            yy += red[BT * VEC + g * per * VEC + c];
          }
          zc[c] = zz;
          st1(op + (size_t)t * HV + cc, yy - ra * zz + rk * ld1(row + 2 * HK + h * dv + cc));
        }
      }
      __syncthreads();
      if (on) {
        float v[VEC], zz[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
          v[e] = ld1(row + 2 * HK + h * dv + strip * VEC + e);
          zz[e] = zc[(tid % per) * VEC + e];
        }
        auto put = [&](int d, float (&xx)[VEC]) {
          const float w = wv[d], k = kv[d], ad = au[d];
#pragma unroll
          for (int e = 0; e < VEC; ++e) xx[e] = fmaf(w, xx[e], fmaf(k, v[e], -ad * zz[e]));
          st_state<NT>(S + strip * VEC + (size_t)d * dv, xx);
        };
        if constexpr (NR > 0) {
#pragma unroll
          for (int i = 0; i < NR; ++i)
            if (rg + i * RG < dk) put(rg + i * RG, x[i]);
        } else {
          for (int d = rg; d < dk; d += RG) {
            get(strip, d, x[0]);
            put(d, x[0]);
          }
        }
      }
      __syncthreads();
    }
  }
}

// A block's matrices.  Elementwise part: a wave takes 16 key channels at a time, lane = (channel l & 15,
// tokens 4 (l >> 4) .. + 3), the accumulator layout of the decay logits.
template <typename E, int NP>
__global__ void __launch_bounds__(256) delta_block_kernel(DeltaArgs a, StepRows r, float* __restrict__ ws) {
  constexpr int NW = 4, LM = 20;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int nb = r.chunk / kBlk, item = blockIdx.x / nb, h = blockIdx.y;
  const int s = r.item_seq[item], ql = r.q_len[s], t0 = r.item_t0[item] + ((int)blockIdx.x % nb) * kBlk;
  const int nt = min(kBlk, ql - t0);
  if (nt <= 0 || s >= r.n_slots) return;  // whole workgroups
  const int dk = a.dk, dkp = delta_dkp(dk), LD = dkp + 4, HK = a.H * dk, HV = a.H * a.dv, rank = a.rank;
  float* Bt = sm;             // [16][LD] each
  float* At = Bt + kBlk * LD;
  float* Kt = At + kBlk * LD;
  float* Rt = Kt + kBlk * LD;
  float* mat = Rt + kBlk * LD;  // [4][16][LM]: T, B~K~, R~K~, R~A~
  float* Xi = mat + 4 * kBlk * LM;  // [16][LM]
  float* red = Xi + kBlk * LM;      // [NW][16]
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, l15 = lane & 15, g4 = lane >> 4;
  const E* proj = reinterpret_cast<const E*>(a.proj) + (size_t)(r.q_start[s] + t0) * a.ldp;
  float* out = ws + ((size_t)blockIdx.x * a.H + h) * delta_per(dkp);
  float* oW = out;
  float* oR = oW + kBlk * dkp;
  float* oK = oR + kBlk * dkp;
  float* oA = oK + kBlk * dkp;
  float* oE = oA + kBlk * dkp;
  float* oM = oE + dkp;

  // every operand's loads first, as stored (the decay projection in steps of 16 RK ranks)
  constexpr int RK = 4;
  E rk[NP][4], rq[NP][4], ra_[NP][4];
  const E* rows[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) rows[i] = proj + (size_t)min(4 * g4 + i, nt - 1) * a.ldp;
  int ch[NP];
  float b0[NP], ab[NP];
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    ch[p] = h * dk + min((p * NW + wid) * 16 + l15, dk - 1);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      rk[p][i] = rows[i][HK + ch[p]];
      rq[p][i] = rows[i][ch[p]];
      ra_[p][i] = rows[i][2 * HK + HV + ch[p]];
    }
    b0[p] = a.w0[ch[p]];
    ab[p] = a.a_b[ch[p]];
  }
  const E* w1 = proj + (size_t)min(l15, nt - 1) * a.ldp + 3 * HK + HV;
  const bool v1 = (3 * HK + HV) % 4 == 0 && a.ldp % 4 == 0 && rank % 4 == 0, v2 = rank % 4 == 0;
  Raw4<E> x1[RK], w2[RK][NP];
  auto fetch = [&](int r0) {
#pragma unroll
    for (int j = 0; j < RK; ++j) {
      const int rc = min(r0 + 16 * j + 4 * g4, v2 ? rank - 4 : rank - 1);
      x1[j].load(w1 + rc, rank - 1 - rc, v1);
#pragma unroll
      for (int p = 0; p < NP; ++p)
        w2[j][p].load(reinterpret_cast<const E*>(a.w2) + (size_t)ch[p] * rank + rc, rank - 1 - rc, v2);
    }
  };
  fetch(0);
  float k[NP][4], rr[NP][4], aa[NP][4];
  float ss[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int d = (p * NW + wid) * 16 + l15;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const bool ok = d < dk && 4 * g4 + i < nt;
      k[p][i] = ok ? ld1(&rk[p][i]) : 0.f;
      rr[p][i] = ok ? ld1(&rq[p][i]) : 0.f;
      aa[p][i] = ok ? ld1(&ra_[p][i]) : 0.f;
      ss[i] = fmaf(k[p][i], k[p][i], ss[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    ss[i] += detail::dpp<0xB1>(ss[i]);
    ss[i] += detail::dpp<0x4E>(ss[i]);
    ss[i] += detail::dpp<0x141>(ss[i]);
    ss[i] += detail::dpp<0x140>(ss[i]);
  }
  if (l15 == 0) *reinterpret_cast<f32x4*>(red + wid * 16 + 4 * g4) = f32x4{ss[0], ss[1], ss[2], ss[3]};
  // decay logits of this wave's channels: rows = tokens, columns = channels
  f32x4 z[NP];
#pragma unroll
  for (int p = 0; p < NP; ++p) z[p] = f32x4{b0[p], b0[p], b0[p], b0[p]};
  for (int r0 = 0; r0 < rank; r0 += 16 * RK) {
    if (r0) fetch(r0);
#pragma unroll
    for (int j = 0; j < RK; ++j) {
      const int left = rank - (r0 + 16 * j + 4 * g4);
      f32x4 x = x1[j].f(left);
#pragma unroll
      for (int i = 0; i < 4; ++i) x[i] = tanh_hw(x[i]);
#pragma unroll
      for (int p = 0; p < NP; ++p) z[p] = mfma_f32x16(x, w2[j][p].f(left), z[p]);
    }
  }
  lds_sync();
  float inv[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    float t = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) t += red[w * 16 + 4 * g4 + i];
    inv[i] = 1.f / sqrtf(t + a.unit_eps);
  }
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int d = (p * NW + wid) * 16 + l15;
    if ((p * NW + wid) * 16 >= dkp) continue;  // whole waves
    float lw[4], b[4], sum = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      lw[i] = (d < dk && 4 * g4 + i < nt) ? log2_decay(a, z[p][i]) : 0.f;
      sum += lw[i];
      b[i] = sum;
    }
    float before = 0.f, all = 0.f;
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      const float x = __shfl(sum, l15 + 16 * g);
      if (g < g4) before += x;
      all += x;
    }
    f32x4 kh, ah;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      b[i] += before;
      const int t = 4 * g4 + i;
      const float u = k[p][i] * inv[i], au = sigmoid_hw(aa[p][i] + ab[p]) * u;
      const float eb = exp2_f(b[i]), en = exp2_f(-b[i]), el = exp2_f(all - b[i]);
      Bt[t * LD + d] = u * exp2_f(b[i] - lw[i]);
      At[t * LD + d] = -au * en;
      Kt[t * LD + d] = k[p][i] * en;
      Rt[t * LD + d] = rr[p][i] * eb;
      kh[i] = k[p][i] * el;
      ah[i] = -au * el;
    }
    *reinterpret_cast<f32x4*>(oK + d * kBlk + 4 * g4) = kh;
    *reinterpret_cast<f32x4*>(oA + d * kBlk + 4 * g4) = ah;
    if (g4 == 0) oE[d] = exp2_f(all);
  }
  lds_sync();
  {  // wave w: one of the four products, row t = 4 g4 + i, column j = l15
    const float* L = (wid < 2 ? Bt : Rt) + l15 * LD + 4 * g4;
    const float* Rr = (wid == 0 || wid == 3 ? At : Kt) + l15 * LD + 4 * g4;
    f32x4 m0 = {0.f, 0.f, 0.f, 0.f}, m1 = m0;
    for (int kt = 0; kt < dkp; kt += 32) {
      m0 = mfma_f32x16(*reinterpret_cast<const f32x4*>(L + kt), *reinterpret_cast<const f32x4*>(Rr + kt), m0);
      if (kt + 16 < dkp)
        m1 = mfma_f32x16(*reinterpret_cast<const f32x4*>(L + kt + 16), *reinterpret_cast<const f32x4*>(Rr + kt + 16), m1);
    }
    m0 += m1;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 4 * g4 + i;
      const bool in = wid < 2 ? l15 < t : l15 <= t;
      mat[(wid * kBlk + t) * LM + l15] = in ? m0[i] : 0.f;
    }
  }
  lds_sync();
  if (wid == 0) {  // column l15 of (I - T)^-1 by forward substitution
    float x[kBlk];
#pragma unroll
    for (int t = 0; t < kBlk; ++t) {
      float acc = t == l15 ? 1.f : 0.f;
#pragma unroll
      for (int c = 0; c < t; ++c) acc = fmaf(mat[t * LM + c], x[c], acc);
      x[t] = acc;
    }
    if (g4 == 0) {
#pragma unroll
      for (int t = 0; t < kBlk; ++t) Xi[t * LM + l15] = x[t];
    }
  }
  lds_sync();
  const f32x4 xi = *reinterpret_cast<const f32x4*>(Xi + l15 * LM + 4 * g4);
  const f32x4 ra = *reinterpret_cast<const f32x4*>(mat + (3 * kBlk + l15) * LM + 4 * g4);
  for (int kt = wid * 16; kt < dkp; kt += NW * 16) {
    f32x4 bt, w = {0.f, 0.f, 0.f, 0.f}, rt;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      bt[i] = Bt[(4 * g4 + i) * LD + kt + l15];
      rt[i] = Rt[(4 * g4 + i) * LD + kt + l15];
    }
    w = mfma_f32x16(xi, bt, w);
    rt = mfma_f32x16(ra, w, rt);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      oW[(4 * g4 + i) * dkp + kt + l15] = w[i];
      oR[(4 * g4 + i) * dkp + kt + l15] = rt[i];
    }
  }
  if (wid == NW - 1) {
    f32x4 mk, m = {0.f, 0.f, 0.f, 0.f}, am;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      mk[i] = mat[(kBlk + 4 * g4 + i) * LM + l15];
      am[i] = mat[(2 * kBlk + 4 * g4 + i) * LM + l15];
    }
    m = mfma_f32x16(xi, mk, m);
    am = mfma_f32x16(ra, m, am);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      oM[(4 * g4 + i) * kBlk + l15] = m[i];
      oM[256 + (4 * g4 + i) * kBlk + l15] = am[i];
    }
  }
}

// DEPTH: blocks whose operands are in registers or on their way
template <typename E, int NW, int KT, int DEPTH>
__global__ void __launch_bounds__(64 * NW) delta_walk_kernel(DeltaArgs a, StepRows r, const float* __restrict__ ws,
                                                             int n_cols) {
  __shared__ __attribute__((aligned(16))) f32x4 part[2][NW][2][64];
  // units: head by head, then portion, then columns: a head's columns read its blocks from one L2
  const int unit = xcd_unit(blockIdx.x, a.H * r.n_crows * n_cols);
  if (unit < 0) return;
  const int h = unit / (r.n_crows * n_cols), crow = unit / n_cols % r.n_crows, s = r.crow_seq[crow];
  if (s >= r.n_slots) return;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, l15 = lane & 15, g4 = lane >> 4;
  const int dk = a.dk, dv = a.dv, dkp = delta_dkp(dk), HK = a.H * dk, HV = a.H * dv;
  const int ql = r.q_len[s], ctx = r.ctx_len[s], q0 = r.q_start[s], nblk = cdiv(ql, kBlk);
  const int col = unit % n_cols * 16 + l15, colc = min(col, dv - 1), n0 = wid * KT * 16;
  const E* vp = reinterpret_cast<const E*>(a.proj) + (size_t)q0 * a.ldp + 2 * HK + h * dv + colc;
  const size_t per = (size_t)delta_per(dkp), stride = per * a.H;
  const float* base = ws + ((size_t)r.crow_item0[crow] * (r.chunk / kBlk) * a.H + h) * per;
  float* st = a.state + ((size_t)s * a.H + h) * dk * dv;

  f32x4 S[KT];
#pragma unroll
  for (int k = 0; k < KT; ++k) {
    S[k] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (ctx != ql && col < dv) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = n0 + 16 * k + 4 * g4 + i;
        if (d < dk) S[k][i] = st[(size_t)d * dv + col];
      }
    }
  }
  struct Ops {
    f32x4 w[KT], r[KT], k[KT], a[KT], e[KT], m, am;
    E v[4];  // (as stored: converting here would wait for every load before)
  };
  // (never conditional: a branch around loads makes every later wait drain them all; past the last block
  // it repeats that one)
  auto fetch = [&](int blk, Ops& o) {
    blk = min(blk, nblk - 1);
    const float* b = base + stride * blk;
#pragma unroll
    for (int k = 0; k < KT; ++k) {
      const int d0 = min(n0 + 16 * k, dkp - 16);  // (tiles past dk: loaded, not used)
      o.w[k] = *reinterpret_cast<const f32x4*>(b + l15 * dkp + d0 + 4 * g4);
      o.r[k] = *reinterpret_cast<const f32x4*>(b + kBlk * dkp + l15 * dkp + d0 + 4 * g4);
      o.k[k] = *reinterpret_cast<const f32x4*>(b + 2 * kBlk * dkp + (d0 + l15) * kBlk + 4 * g4);
      o.a[k] = *reinterpret_cast<const f32x4*>(b + 3 * kBlk * dkp + (d0 + l15) * kBlk + 4 * g4);
      o.e[k] = *reinterpret_cast<const f32x4*>(b + 4 * kBlk * dkp + d0 + 4 * g4);
    }
    const float* m = b + 65l * dkp;
    o.m = *reinterpret_cast<const f32x4*>(m + l15 * kBlk + 4 * g4);
    o.am = *reinterpret_cast<const f32x4*>(m + 256 + l15 * kBlk + 4 * g4);
#pragma unroll
    for (int i = 0; i < 4; ++i) o.v[i] = vp[(size_t)min(blk * kBlk + 4 * g4 + i, ql - 1) * a.ldp];
  };
  auto step = [&](int blk, const Ops& o, Ops& fill) {
    fetch(blk + DEPTH - 1, fill);
    const int buf = blk & 1;
    const f32x4 v = {ld1(&o.v[0]), ld1(&o.v[1]), ld1(&o.v[2]), ld1(&o.v[3])};
    f32x4 x = {0.f, 0.f, 0.f, 0.f}, y = x;
    if (wid == 0) {
      x = mfma_f32x16(o.m, v, x);
      y = mfma_f32x16(o.am, v, y);
    }
#pragma unroll
    for (int k = 0; k < KT; ++k) {
      if (n0 + 16 * k < dkp) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          x = mfma_f32(o.w[k][i], S[k][i], x);
          y = mfma_f32(o.r[k][i], S[k][i], y);
        }
      }
    }
    part[buf][wid][0][lane] = x;
    part[buf][wid][1][lane] = y;
#pragma unroll
    for (int k = 0; k < KT; ++k)
      if (n0 + 16 * k < dkp) S[k] = mfma_f32x16(o.k[k], v, S[k] * o.e[k]);
    lds_sync();
    x = part[buf][0][0][lane];
#pragma unroll
    for (int w = 1; w < NW; ++w) x += part[buf][w][0][lane];
#pragma unroll
    for (int k = 0; k < KT; ++k)
      if (n0 + 16 * k < dkp) S[k] = mfma_f32x16(o.a[k], x, S[k]);
    if ((blk & (NW - 1)) == wid) {  // the waves take the outputs in turn
      y = part[buf][0][1][lane];
#pragma unroll
      for (int w = 1; w < NW; ++w) y += part[buf][w][1][lane];
      E* out = reinterpret_cast<E*>(a.o) + (size_t)(q0 + blk * kBlk) * HV + h * dv + col;
      if (col < dv) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (blk * kBlk + 4 * g4 + i < ql) st1(out + (size_t)(4 * g4 + i) * HV, y[i]);
      }
    }
  };
  Ops o[DEPTH];
#pragma unroll
  for (int j = 0; j < DEPTH - 1; ++j) fetch(j, o[j]);
  int blk = 0;
  for (; blk + DEPTH <= nblk; blk += DEPTH) {
#pragma unroll
    for (int j = 0; j < DEPTH; ++j) step(blk + j, o[j], o[(j + DEPTH - 1) % DEPTH]);
  }
#pragma unroll
  for (int j = 0; j < DEPTH - 1; ++j)
    if (blk + j < nblk) step(blk + j, o[j], o[(j + DEPTH - 1) % DEPTH]);
#pragma unroll
  for (int k = 0; k < KT; ++k)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = n0 + 16 * k + 4 * g4 + i;
      if (d < dk && col < dv) st[(size_t)d * dv + col] = S[k][i];
    }
}

template <typename E, int VEC, int BT>
static void delta_rows_nr(const DeltaArgs& a, const StepRows& s, const int* rows, int n, hipStream_t st) {
  const int per = std::min(a.dv / VEC, BT), rg = BT / per, nr = cdiv(a.dk, rg);
  const size_t lds = (size_t)(a.rank + 5 * a.dk + 3 * BT * VEC) * 4;
  const dim3 grid(n, a.H);
  const bool nt = (size_t)n * a.H * a.dk * a.dv * 4 >= kStreamBytes;
#define MLOP_ROWS(NR)                                                                       \
  do {                                                                                      \
    if (nt) delta_rows_kernel<E, VEC, BT, NR, true><<<grid, BT, lds, st>>>(a, s, rows);     \
    else delta_rows_kernel<E, VEC, BT, NR, false><<<grid, BT, lds, st>>>(a, s, rows);       \
  } while (0)
  if (nr > 16 || a.dv / VEC > BT) MLOP_ROWS(0);
  else if (nr <= 4) MLOP_ROWS(4);
  else MLOP_ROWS(16);
#undef MLOP_ROWS
}

template <typename E>
static void delta_rows(const DeltaArgs& a, const StepRows& s, const int* rows, int n, hipStream_t st) {
  if (n == 0) return;
  if (a.dv % 4) return delta_rows_nr<E, 1, 256>(a, s, rows, n, st);
  // few (row, head) pairs: a whole CU's threads on each, so that its state is in flight at once
  if (n * a.H <= 256 && (long)a.dk * a.dv >= 8192) delta_rows_nr<E, 4, 512>(a, s, rows, n, st);
  else delta_rows_nr<E, 4, 256>(a, s, rows, n, st);
}

template <typename E, int NP>
static void delta_blocks(const DeltaArgs& a, const StepRows& s, float* ws, hipStream_t st) {
  const int dkp = delta_dkp(a.dk);
  const size_t lds = (size_t)(4 * kBlk * (dkp + 4) + 5 * kBlk * 20 + 4 * 16) * 4;
  auto k = delta_block_kernel<E, NP>;
  static bool attr = false;
  if (!attr && lds > 65536) {
    (void)hipFuncSetAttribute((const void*)k, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    attr = true;
  }
  k<<<dim3(s.n_items * (s.chunk / kBlk), a.H), 256, lds, st>>>(a, s, ws);
}

template <typename E>
static void delta_all(const DeltaArgs& a, const StepRows& s, float* ws, hipStream_t st) {
  delta_rows<E>(a, s, s.rows, s.n_rows, st);
  if (s.n_crows == 0) return;
  if (!delta_blocks_ok(a.dk, a.decay_scale)) return delta_rows<E>(a, s, s.crow_seq, s.n_crows, st);
  const int cols = cdiv(a.dv, 16), grid = xcd_grid(a.H * s.n_crows * cols);
  if (a.dk <= 64) {
    delta_blocks<E, 1>(a, s, ws, st);
    delta_walk_kernel<E, 4, 1, 3><<<grid, 256, 0, st>>>(a, s, ws, cols);
  } else if (a.dk <= 128) {
    delta_blocks<E, 2>(a, s, ws, st);
    // few units: more waves on each (latency); many: fewer, with more in flight per CU
    if (grid < 1024) delta_walk_kernel<E, 8, 1, 3><<<grid, 512, 0, st>>>(a, s, ws, cols);
    else delta_walk_kernel<E, 4, 2, 2><<<grid, 256, 0, st>>>(a, s, ws, cols);
  } else {
    delta_blocks<E, 4>(a, s, ws, st);
    delta_walk_kernel<E, 8, 2, 2><<<grid, 512, 0, st>>>(a, s, ws, cols);
  }
}

bool delta_blocks_ok(int dk, float decay_scale) { return dk <= kDeltaMaxDk && decay_scale * kBlk <= kMaxBlockDecay; }

long delta_ws_floats(int n_items, int chunk, int H, int dk) {
  return (long)n_items * (chunk / kBlk) * H * delta_per(delta_dkp(dk));
}

void launch_delta(const DeltaArgs& a, const StepRows& s, float* ws, bool f32, hipStream_t st) {
  if (f32) delta_all<float>(a, s, ws, st);
  else delta_all<uint16_t>(a, s, ws, st);
}

}  // namespace mlop
