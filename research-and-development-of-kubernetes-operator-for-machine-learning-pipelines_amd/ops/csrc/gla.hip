// Gated linear attention: per head a matrix state S [dk, dv] in fp32, carried from token to token,
//
//   S_t = diag(exp(g_t)) S_{t-1} + k_t v_t^T        o_t = S_t^T q_t
//   g_t = log(sigmoid(z_t)) / tau,  z_t = A2 a1_t + b    (one log-decay per key channel, <= 0)
//
// then each head's o RMS-normed over dv, times silu(gate).  Everything of the recurrence is fp32
// (the projections arrive in the model dtype); the matrix products use the fp32 MFMA.
//
// Two forms, chosen by a row's tokens in the step:
//   gla_rows_kernel   one token (any number, one after the other): a workgroup per (row, head)
//                     streams the state once, HBM-bound, with decay, norm and gate in the launch;
//   gla_chunk_*       prompt chunks of C tokens in parallel: (1) every chunk's own contribution to
//                     the state and its total decay, (2) an elementwise scan over a sequence's
//                     chunks that turns them into each chunk's starting state and leaves the last
//                     one in the state cache, (3) the outputs, in blocks of 16 tokens.
// With b_t the running sum of g inside a block of 16 tokens, the block's outputs are
//   o_t = (q_t e^{b_t})^T S + sum_{j <= t} [ sum_d q_td k_jd e^{b_td - b_jd} ] v_j
// and its state update S <- diag(e^{b_16}) S + sum_j (k_j e^{b_16 - b_j}) v_j^T: every exponent is
// <= 0.  The score factorises as (q e^b) (k e^-b) for the MFMA while no channel decays by more than
// e^-60 in a block (all in fp32 range); else it is summed pair by pair with the exponents <= 0.
//
// A sequence's first token (context length = tokens of this step) starts from the zero state
// whatever its slot holds, so slots need no clearing when they are handed on.
#include "elem.h"
#include "hybrid.h"

namespace mlop {

namespace {

constexpr float kFastDecay = -60.f;

__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float silu_f(float x) { return x / (1.f + expf(-x)); }
__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) {
  // lane l: A[row l & 15][k = l >> 4], B[k = l >> 4][col l & 15]; C/D row 4 (l >> 4) + i, col l & 15
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// z of key channel n (a row of A2) for the a1 vector in LDS / registers
template <typename E>
__device__ __forceinline__ float decay_logit(const GlaArgs& a, int n, const float* a1) {
  const E* w = reinterpret_cast<const E*>(a.a2) + (size_t)n * a.rank;
  float z = a.a2_b[n];
  for (int i = 0; i < a.rank; ++i) z = fmaf(ld1(w + i), a1[i], z);
  return z;
}

}  // namespace

// Workgroup = (row, head).  Threads own VEC-column strips: strip s = tid % strips, key rows
// rg, rg + RG, ... with rg = tid / strips.
template <typename E, int VEC, int BT>
__global__ void __launch_bounds__(BT) gla_rows_kernel(GlaArgs a, const int* __restrict__ rows) {
  extern __shared__ float sm[];
  __shared__ float scratch[16];
  const int s = rows[blockIdx.x], h = blockIdx.y, tid = threadIdx.x;
  const int dk = a.dk, dv = a.dv;
  float* a1 = sm;                  // [rank]
  float* dec = a1 + a.rank;        // [dk]
  float* q = dec + dk;             // [dk]
  float* k = q + dk;               // [dk]
  float* o = k + dk;               // [dv]
  float* red = o + dv;             // [BT * VEC]
  const int ql = a.q_len[s], ctx = a.ctx_len[s], qs = a.q_start[s];
  E* outp = reinterpret_cast<E*>(a.out);
  if (ctx < ql || s >= a.n_slots) {  // graph padding: attends to nothing, holds no state
    for (int t = 0; t < ql; ++t)
      for (int c = tid; c < dv; c += BT) st1(outp + ((size_t)(qs + t) * a.H + h) * dv + c, 0.f);
    return;
  }
  float* S = a.state + ((size_t)s * a.H + h) * dk * dv;
  const int nstrip = dv / VEC, per = min(nstrip, BT), RG = BT / per;
  const int HK = a.H * dk, HV = a.H * dv;
  for (int t = 0; t < ql; ++t) {
    const E* row = reinterpret_cast<const E*>(a.proj) + (size_t)(qs + t) * a.ldp;
    const bool fresh = ctx - ql + t == 0;
    for (int i = tid; i < a.rank; i += BT) a1[i] = ld1(row + 2 * HK + 2 * HV + i);
    __syncthreads();
    for (int d = tid; d < dk; d += BT) {
      dec[d] = expf(log_sigmoid(decay_logit<E>(a, h * dk + d, a1)) * a.inv_tau);
      q[d] = ld1(row + h * dk + d) * a.q_scale;
      k[d] = ld1(row + HK + h * dk + d);
    }
    __syncthreads();
    for (int s0 = 0; s0 < nstrip; s0 += per) {
      const int strip = s0 + tid % per, rg = tid / per;
      float acc[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) acc[e] = 0.f;
      if (rg < RG && strip < nstrip) {
        float v[VEC];
        const E* vp = row + 2 * HK + h * dv + strip * VEC;
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] = ld1(vp + e);
        float* col = S + strip * VEC;
#pragma unroll BT >= 1024 ? 4 : 8
        for (int d = rg; d < dk; d += RG) {
          float x[VEC];
          if (fresh) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) x[e] = 0.f;
          } else {
            ldn<VEC>(col + (size_t)d * dv, x);
          }
          const float de = dec[d], kd = k[d], qd = q[d];
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            x[e] = fmaf(de, x[e], kd * v[e]);
            acc[e] = fmaf(qd, x[e], acc[e]);
          }
          stn<VEC>(col + (size_t)d * dv, x);
        }
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) red[tid * VEC + e] = acc[e];
      __syncthreads();
      for (int c = tid; c < per * VEC; c += BT) {
        if (s0 * VEC + c < dv) {
          float x = 0.f;
          for (int g = 0; g < RG; ++g) x += red[g * per * VEC + c];
          o[s0 * VEC + c] = x;
        }
      }
      __syncthreads();
    }
    float ss = 0.f;
    for (int c = tid; c < dv; c += BT) ss = fmaf(o[c], o[c], ss);
    ss = block_sum(ss, scratch);
    const float inv = 1.f / sqrtf(ss / (float)dv + a.eps);
    const E* gp = row + 2 * HK + HV + h * dv;
    for (int c = tid; c < dv; c += BT)
      st1(outp + ((size_t)(qs + t) * a.H + h) * dv + c, o[c] * inv * a.norm_w[c] * silu_f(ld1(gp + c)));
  }
}

// One chunk of one head for a group of 128 NCT value columns; 8 waves.
//   OUT = false: the chunk's own contribution from a zero state -> cstate, total decay -> cdecay
//   OUT = true:  outputs from the chunk's starting state in cstate: normed and gated straight to `out`
//                when the group holds the whole head (dv <= 128 NCT), else raw to o32
// Elementwise part: a wave takes 16 key channels at a time, lane = (channel l & 15, tokens
// 4 (l >> 4) .. + 3) -- the accumulator layout of z = a1 A2^T, which the MFMA computes in place.  The
// decays live in the log2 domain.  Products: wave w owns 16 NCT value columns, the state
// [16 NKT, 16 NCT] in its accumulators.
constexpr int kGlaWaves = 8;

// workgroup barrier for LDS hand-offs only: outstanding global loads (the next block's operands) and
// stores stay in flight across it, which __syncthreads would wait for
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  raw_barrier();
}

__device__ __forceinline__ float exp2_g(float x) { return __builtin_amdgcn_exp2f(x); }
// log2(sigmoid(z)): log1p by the quotient form, exact where 1 + e rounds
__device__ __forceinline__ float log2_sigmoid(float z) {
  const float e = exp2_g(-fabsf(z) * 1.44269504f), u = 1.f + e, d = u - 1.f;
  const float l = d == 0.f ? e * 1.44269504f : __builtin_amdgcn_logf(u) * (e * __builtin_amdgcn_rcpf(d));
  return fminf(z, 0.f) * 1.44269504f - l;
}

// waves per SIMD the chunk kernel is built for: 4 = two workgroups per CU (128 VGPRs), 2 = one
constexpr int chunk_waves(int nkt, int nct, bool out) {
  return (nct == 1 ? nkt <= 8 : !out && nkt <= 4) ? 4 : 2;
}

template <typename E, int NKT, int NCT, bool OUT>
__global__ void __launch_bounds__(64 * kGlaWaves, chunk_waves(NKT, NCT, OUT)) gla_chunk_kernel(
    GlaArgs a, float* __restrict__ o32, float* __restrict__ cstate, float* __restrict__ cdecay,
    const int* __restrict__ item_seq, const int* __restrict__ item_t0, int chunk) {
  constexpr int NW = kGlaWaves, DKP = 16 * NKT, LD = DKP + 4, LT = 20, NP = (NKT + NW - 1) / NW;
  constexpr float kFast2 = kFastDecay * 1.44269504f;
  // operands fetched one block ahead where the registers allow it at two workgroups per CU
  constexpr bool AHEAD = NKT * NCT <= (chunk_waves(NKT, NCT, OUT) == 2 ? 16 : OUT ? 2 : 8);
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* KT = sm;                     // [DKP][LT]: k_j e^{b_16 - b_j}, token fastest
  float* En = KT + DKP * LT;          // [DKP]: e^{b_16}
  float* Qs = En + DKP;               // [16][LD]: q e^b            (OUT only from here on)
  float* Ks = Qs + 16 * LD;           // [16][LD]: k e^-b
  float* part = Ks + 16 * LD;         // [NW][256]
  float* red = part + NW * 256;       // [NW][16]
  float* flags = red + NW * 16;       // [2][NW]
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int item = blockIdx.x, h = blockIdx.y;
  const int s = item_seq[item], t0 = item_t0[item];
  const int n = min(chunk, a.q_len[s] - t0), tok0 = a.q_start[s] + t0;
  const int dk = a.dk, dv = a.dv, HK = a.H * dk, HV = a.H * dv, rank = a.rank;
  const int l15 = lane & 15, g4 = lane >> 4;
  const int col0 = ((int)blockIdx.z * NW + wid) * 16 * NCT;  // first column of this wave
  const bool wave_cols = col0 < dv;
  const bool fused = OUT && gridDim.z == 1;
  const E* proj = reinterpret_cast<const E*>(a.proj) + (size_t)tok0 * a.ldp;
  const E* pa = proj + 2 * HK + 2 * HV;
  float* cst = cstate + ((size_t)item * a.H + h) * dk * dv;

  f32x4 S[NKT][NCT];
#pragma unroll
  for (int kt = 0; kt < NKT; ++kt)
#pragma unroll
    for (int c = 0; c < NCT; ++c) {
      S[kt][c] = f32x4{0.f, 0.f, 0.f, 0.f};
      const int col = col0 + 16 * c + l15;
      if (OUT && col < dv) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int d = 16 * kt + 4 * g4 + i;
          if (d < dk) S[kt][c][i] = cst[(size_t)d * dv + col];
        }
      }
    }
  float nw[NCT];
#pragma unroll
  for (int c = 0; c < NCT; ++c) nw[c] = (fused && col0 + 16 * c + l15 < dv) ? a.norm_w[col0 + 16 * c + l15] : 0.f;
  const float inv_dv = 1.f / (float)dv;
  float total[NP];
#pragma unroll
  for (int p = 0; p < NP; ++p) total[p] = 0.f;

  // A block's operands as stored: loads at clamped addresses, unconditional and not converted here, so
  // that all of them are in flight together; `take` converts and zeroes what is out of range.
  E rk[NP][4], rq[NP][4], rv[NCT][4], rg[NCT][4], rx[4];
  auto fetch = [&](int t) {
    const E* rows[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) rows[i] = proj + (size_t)min(t + 4 * g4 + i, n - 1) * a.ldp;
    const E* xrow = proj + (size_t)min(t + l15, n - 1) * a.ldp + 2 * HK + 2 * HV;
#pragma unroll
    for (int i = 0; i < 4; ++i) rx[i] = xrow[min(4 * g4 + i, rank - 1)];
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      const int d = h * dk + min((p * NW + wid) * 16 + l15, dk - 1);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        rk[p][i] = rows[i][HK + d];
        if (OUT) rq[p][i] = rows[i][d];
      }
    }
#pragma unroll
    for (int c = 0; c < NCT; ++c) {
      const int v = 2 * HK + h * dv + min(col0 + 16 * c + l15, dv - 1);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        rv[c][i] = rows[i][v];
        if (OUT) rg[c][i] = rows[i][HV + v];
      }
    }
  };
  float kk[NP][4], qq[NP][4], cv[NCT][4], gg[NCT][4], x1[4];
  auto take = [&](int nt) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const bool in = 4 * g4 + i < nt;
      x1[i] = (l15 < nt && 4 * g4 + i < rank) ? ld1(&rx[i]) : 0.f;
#pragma unroll
      for (int p = 0; p < NP; ++p) {
        const bool ok = in && (p * NW + wid) * 16 + l15 < dk;
        kk[p][i] = ok ? ld1(&rk[p][i]) : 0.f;
        if (OUT) qq[p][i] = ok ? ld1(&rq[p][i]) * a.q_scale : 0.f;
      }
#pragma unroll
      for (int c = 0; c < NCT; ++c) {
        cv[c][i] = (in && col0 + 16 * c + l15 < dv) ? ld1(&rv[c][i]) : 0.f;
        if (OUT) gg[c][i] = ld1(&rg[c][i]);
      }
    }
  };
  // this wave's rows of A2 (its first 16 columns) and biases, kept over the chunk: a load inside the
  // loop would wait behind the previous block's stores
  float w1[NP][4], bias[NP];
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int d = (p * NW + wid) * 16 + l15, nrow = h * dk + (d < dk ? d : 0);
    bias[p] = a.a2_b[nrow];
#pragma unroll
    for (int i = 0; i < 4; ++i)
      w1[p][i] = 4 * g4 + i < rank ? ld1(reinterpret_cast<const E*>(a.a2) + (size_t)nrow * rank + 4 * g4 + i) : 0.f;
  }
  if (AHEAD) fetch(0);
  for (int t = 0; t < n; t += 16) {
    const int nt = min(16, n - t);
    if (!AHEAD) fetch(t);
    take(nt);
    if (AHEAD && t + 16 < n) fetch(t + 16);
    // log2 decays of this wave's channels, running sums over the block's tokens
    float b[NP][4], bn[NP];
    bool slow = false;
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      const int d = (p * NW + wid) * 16 + l15;
      const bool ok = d < dk;
      f32x4 z = {bias[p], bias[p], bias[p], bias[p]};
#pragma unroll
      for (int i = 0; i < 4; ++i) z = mfma4(x1[i], w1[p][i], z);
      const E* w = reinterpret_cast<const E*>(a.a2) + (size_t)(h * dk + (ok ? d : 0)) * rank;
      for (int r0 = 16; r0 < rank; r0 += 16) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int r = r0 + 4 * g4 + i;
          const float x = (l15 < nt && r < rank) ? ld1(pa + (size_t)(t + l15) * a.ldp + r) : 0.f;
          z = mfma4(x, r < rank ? ld1(w + r) : 0.f, z);
        }
      }
      float sum = 0.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if (ok && 4 * g4 + i < nt) sum += log2_sigmoid(z[i]) * a.inv_tau;
        b[p][i] = sum;
      }
      float before = 0.f, all = 0.f;
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        const float x = __shfl(sum, l15 + 16 * g);
        if (g < g4) before += x;
        all += x;
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) b[p][i] += before;
      bn[p] = all;
      total[p] += all;
      slow |= all < kFast2;
    }
    bool fast = true;
    if (OUT) {
      float* fl = flags + (t & 16 ? NW : 0);
      const bool any = __ballot(slow) != 0;
      if (lane == 0) fl[wid] = any ? 1.f : 0.f;
      lds_barrier();  // also: the last block's LDS reads are done
      float f = 0.f;
#pragma unroll
      for (int w = 0; w < NW; ++w) f += fl[w];
      fast = f == 0.f;
    } else {
      lds_barrier();
    }
    auto put_kt = [&]() {
#pragma unroll
      for (int p = 0; p < NP; ++p) {
        const int d = (p * NW + wid) * 16 + l15;
        if (d < DKP)
          *reinterpret_cast<f32x4*>(KT + d * LT + 4 * g4) =
              f32x4{kk[p][0] * exp2_g(bn[p] - b[p][0]), kk[p][1] * exp2_g(bn[p] - b[p][1]),
                    kk[p][2] * exp2_g(bn[p] - b[p][2]), kk[p][3] * exp2_g(bn[p] - b[p][3])};
      }
    };
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      const int d = (p * NW + wid) * 16 + l15;
      if (d < DKP) {
        if (g4 == 0) En[d] = exp2_g(bn[p]);
        if (OUT) {
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int j = 4 * g4 + i;
            Qs[j * LD + d] = fast ? qq[p][i] * exp2_g(b[p][i]) : qq[p][i];
            Ks[j * LD + d] = fast ? kk[p][i] * exp2_g(-b[p][i]) : kk[p][i];
            if (!fast) KT[j * LD + d] = b[p][i];  // (DKP * LT >= 16 * LD)
          }
        }
      }
    }
    if (!OUT || fast) put_kt();
    lds_barrier();
    f32x4 A = {0.f, 0.f, 0.f, 0.f};  // scores^T: row j = 4 g4 + i, column = token l15
    if (OUT) {
      int nsum = min(NW, NKT);
      if (fast) {
        f32x4 sc = {0.f, 0.f, 0.f, 0.f};
        for (int kt = wid; kt < NKT; kt += NW) {
          const f32x4 x = *reinterpret_cast<const f32x4*>(Ks + l15 * LD + 16 * kt + 4 * g4);
          const f32x4 y = *reinterpret_cast<const f32x4*>(Qs + l15 * LD + 16 * kt + 4 * g4);
#pragma unroll
          for (int i = 0; i < 4; ++i) sc = mfma4(x[i], y[i], sc);
        }
        if (wid < NKT) {
#pragma unroll
          for (int i = 0; i < 4; ++i) part[wid * 256 + (4 * g4 + i) * 16 + l15] = sc[i];
        }
      } else {
        nsum = 2;
        const int half = tid >> 8, j = (tid >> 4) & 15, tt = tid & 15;
        float x = 0.f;
        if (j <= tt)
          for (int d = half; d < dk; d += 2)
            x = fmaf(Qs[tt * LD + d] * Ks[j * LD + d], exp2_g(KT[tt * LD + d] - KT[j * LD + d]), x);
        part[tid] = x;
        lds_barrier();
#pragma unroll
        for (int p = 0; p < NP; ++p) {
          const int d = (p * NW + wid) * 16 + l15;
          if (d < DKP) {
#pragma unroll
            for (int i = 0; i < 4; ++i) Qs[(4 * g4 + i) * LD + d] = qq[p][i] * exp2_g(b[p][i]);
          }
        }
        put_kt();
      }
      lds_barrier();
      for (int w = 0; w < nsum; ++w)
#pragma unroll
        for (int i = 0; i < 4; ++i) A[i] += part[w * 256 + (4 * g4 + i) * 16 + l15];
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (4 * g4 + i > l15) A[i] = 0.f;
    }
    f32x4 o[NCT];
    if (OUT) {
#pragma unroll
      for (int c = 0; c < NCT; ++c) {
        o[c] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < 4; ++i) o[c] = mfma4(A[i], cv[c][i], o[c]);
      }
      if (wave_cols) {
#pragma unroll
        for (int kt = 0; kt < NKT; ++kt) {
          const f32x4 y = *reinterpret_cast<const f32x4*>(Qs + l15 * LD + 16 * kt + 4 * g4);
#pragma unroll
          for (int c = 0; c < NCT; ++c)
#pragma unroll
            for (int i = 0; i < 4; ++i) o[c] = mfma4(y[i], S[kt][c][i], o[c]);
        }
      }
    }
    if (wave_cols && (!OUT || t + 16 < n)) {
#pragma unroll
      for (int kt = 0; kt < NKT; ++kt) {
        const f32x4 e = *reinterpret_cast<const f32x4*>(En + 16 * kt + 4 * g4);
        const f32x4 x = *reinterpret_cast<const f32x4*>(KT + (16 * kt + l15) * LT + 4 * g4);
#pragma unroll
        for (int c = 0; c < NCT; ++c) {
          S[kt][c] *= e;
#pragma unroll
          for (int i = 0; i < 4; ++i) S[kt][c] = mfma4(x[i], cv[c][i], S[kt][c]);
        }
      }
    }
    if (fused) {  // o row 4 g4 + i = token, over the head's columns: rms, weight, gate
      float ss[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        ss[i] = 0.f;
#pragma unroll
        for (int c = 0; c < NCT; ++c) ss[i] = fmaf(o[c][i], o[c][i], ss[i]);  // columns past dv are zero
        ss[i] += detail::dpp<0xB1>(ss[i]);
        ss[i] += detail::dpp<0x4E>(ss[i]);
        ss[i] += detail::dpp<0x141>(ss[i]);
        ss[i] += detail::dpp<0x140>(ss[i]);
      }
      if (l15 == 0) *reinterpret_cast<f32x4*>(red + wid * 16 + 4 * g4) = f32x4{ss[0], ss[1], ss[2], ss[3]};
      lds_barrier();
      f32x4 tot = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int w = 0; w < NW; ++w) tot += *reinterpret_cast<const f32x4*>(red + w * 16 + 4 * g4);
      E* op = reinterpret_cast<E*>(a.out) + (size_t)(tok0 + t) * HV + h * dv;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int j = 4 * g4 + i;
        const float inv = rsqrtf(tot[i] * inv_dv + a.eps);
#pragma unroll
        for (int c = 0; c < NCT; ++c) {
          const int col = col0 + 16 * c + l15;
          if (col < dv && j < nt) {
            const float g = gg[c][i];
            st1(op + (size_t)j * HV + col, o[c][i] * inv * nw[c] * (g * __builtin_amdgcn_rcpf(1.f + exp2_g(-g * 1.44269504f))));
          }
        }
      }
    } else if (OUT) {
#pragma unroll
      for (int c = 0; c < NCT; ++c)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int j = 4 * g4 + i, col = col0 + 16 * c + l15;
          if (col < dv && j < nt) o32[(size_t)(tok0 + t + j) * HV + h * dv + col] = o[c][i];
        }
    }
  }
  if (!OUT) {
#pragma unroll
    for (int kt = 0; kt < NKT; ++kt)
#pragma unroll
      for (int c = 0; c < NCT; ++c)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int d = 16 * kt + 4 * g4 + i, col = col0 + 16 * c + l15;
          if (d < dk && col < dv) cst[(size_t)d * dv + col] = S[kt][c][i];
        }
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      const int d = (p * NW + wid) * 16 + l15;
      if (d < dk && g4 == 0 && blockIdx.z == 0) cdecay[((size_t)item * a.H + h) * dk + d] = exp2_g(total[p]);
    }
  }
}

// cstate[item] <- state in front of the item's chunk; the state cache <- behind the last chunk
__global__ void __launch_bounds__(256) gla_scan_kernel(GlaArgs a, float* __restrict__ cstate,
                                                       const float* __restrict__ cdecay,
                                                       const int* __restrict__ crow_seq,
                                                       const int* __restrict__ crow_item0, int chunk) {
  const int s = crow_seq[blockIdx.x], i0 = crow_item0[blockIdx.x], h = blockIdx.y;
  const int ql = a.q_len[s], n = (ql + chunk - 1) / chunk;
  const int e = blockIdx.z * 256 + threadIdx.x, sz = a.dk * a.dv;
  if (e >= sz || s >= a.n_slots) return;
  const int d = e / a.dv;
  float* st = a.state + ((size_t)s * a.H + h) * sz + e;
  float x = a.ctx_len[s] == ql ? 0.f : *st;
  float* c = cstate + ((size_t)i0 * a.H + h) * sz + e;
  const float* dc = cdecay + ((size_t)i0 * a.H + h) * a.dk + d;
  const size_t cs = (size_t)a.H * sz, ds = (size_t)a.H * a.dk;
#pragma unroll 4
  for (int i = 0; i < n; ++i) {
    const float add = c[i * cs], f = dc[i * ds];
    c[i * cs] = x;
    x = fmaf(f, x, add);
  }
  *st = x;
}

// out <- o32 / rms(o32 over dv) * norm_w * silu(g): a wave per (token of an item, head)
template <typename E>
__global__ void __launch_bounds__(256) gla_gate_kernel(GlaArgs a, const float* __restrict__ o32,
                                                       const int* __restrict__ item_seq,
                                                       const int* __restrict__ item_t0, int chunk) {
  const int s = item_seq[blockIdx.x], t0 = item_t0[blockIdx.x], lane = threadIdx.x & 63;
  const int n = min(chunk, a.q_len[s] - t0), w = blockIdx.y * 4 + (threadIdx.x >> 6);
  const int t = w / a.H, h = w - t * a.H;
  if (t >= n) return;  // whole waves
  const size_t tok = a.q_start[s] + t0 + t;
  const float* o = o32 + (tok * a.H + h) * a.dv;
  const E* g = reinterpret_cast<const E*>(a.proj) + tok * a.ldp + 2 * a.H * a.dk + a.H * a.dv + h * a.dv;
  E* out = reinterpret_cast<E*>(a.out) + (tok * a.H + h) * a.dv;
  float ss = 0.f;
  for (int c = lane; c < a.dv; c += 64) ss = fmaf(o[c], o[c], ss);
  const float inv = 1.f / sqrtf(wave_sum(ss) / (float)a.dv + a.eps);
  for (int c = lane; c < a.dv; c += 64) st1(out + c, o[c] * inv * a.norm_w[c] * silu_f(ld1(g + c)));
}

template <typename E, int BT>
static void run_rows_t(const GlaArgs& a, const int* rows, int n_rows, hipStream_t st) {
  const bool v4 = a.dv % 4 == 0;
  const size_t lds = (size_t)(a.rank + 3 * a.dk + a.dv + BT * (v4 ? 4 : 1)) * 4;
  if (v4) gla_rows_kernel<E, 4, BT><<<dim3(n_rows, a.H), BT, lds, st>>>(a, rows);
  else gla_rows_kernel<E, 1, BT><<<dim3(n_rows, a.H), BT, lds, st>>>(a, rows);
}

template <typename E>
static void run_rows(const GlaArgs& a, const int* rows, int n_rows, hipStream_t st) {
  // few (row, head) pairs: a whole CU's threads on each, so that its state is in flight at once
  if (n_rows * a.H <= 256 && (long)a.dk * a.dv >= 8192) run_rows_t<E, 1024>(a, rows, n_rows, st);
  else run_rows_t<E, 256>(a, rows, n_rows, st);
}

void launch_gla_rows(const GlaArgs& a, bool f32, const int* rows, int n_rows, hipStream_t st) {
  if (n_rows == 0) return;
  if (f32) run_rows<float>(a, rows, n_rows, st);
  else run_rows<uint16_t>(a, rows, n_rows, st);
}

template <typename E, int NKT, int NCT>
static void run_chunks(const GlaArgs& a, float* o32, float* cstate, float* cdecay, const int* item_seq,
                       const int* item_t0, int n_items, const int* crow_seq, const int* crow_item0, int n_crows,
                       int chunk, hipStream_t st) {
  const dim3 grid(n_items, a.H, cdiv(a.dv, 16 * kGlaWaves * NCT));
  constexpr int DKP = 16 * NKT, LD = DKP + 4;
  constexpr size_t lds1 = (size_t)(DKP * 20 + DKP) * 4;
  constexpr size_t lds2 = lds1 + (size_t)(2 * 16 * LD + kGlaWaves * (256 + 16 + 2)) * 4;
  auto k1 = gla_chunk_kernel<E, NKT, NCT, false>;
  auto k2 = gla_chunk_kernel<E, NKT, NCT, true>;
  static bool attr = false;
  if (!attr && lds2 > 65536) {
    (void)hipFuncSetAttribute((const void*)k2, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds2);
    attr = true;
  }
  k1<<<grid, 64 * kGlaWaves, lds1, st>>>(a, nullptr, cstate, cdecay, item_seq, item_t0, chunk);
  gla_scan_kernel<<<dim3(n_crows, a.H, cdiv(a.dk * a.dv, 256)), 256, 0, st>>>(a, cstate, cdecay, crow_seq, crow_item0,
                                                                              chunk);
  k2<<<grid, 64 * kGlaWaves, lds2, st>>>(a, o32, cstate, cdecay, item_seq, item_t0, chunk);
  if (grid.z > 1)
    gla_gate_kernel<E><<<dim3(n_items, cdiv(chunk * a.H, 4)), 256, 0, st>>>(a, o32, item_seq, item_t0, chunk);
}

bool gla_chunks_need_o32(int dv) { return dv > 2 * 16 * kGlaWaves; }

void launch_gla_chunks(const GlaArgs& a, bool f32, float* o32, float* cstate, float* cdecay, const int* item_seq,
                       const int* item_t0, int n_items, const int* crow_seq, const int* crow_item0, int n_crows,
                       int chunk, hipStream_t st) {
  if (n_items == 0) return;
#define MLOP_GLA_C(N, C)                                                                                          \
  do {                                                                                                            \
    if (f32) run_chunks<float, N, C>(a, o32, cstate, cdecay, item_seq, item_t0, n_items, crow_seq, crow_item0,    \
                                     n_crows, chunk, st);                                                         \
    else run_chunks<uint16_t, N, C>(a, o32, cstate, cdecay, item_seq, item_t0, n_items, crow_seq, crow_item0,     \
                                    n_crows, chunk, st);                                                          \
  } while (0)
#define MLOP_GLA(N)                                                        \
  do {                                                                     \
    if (a.dv <= 16 * kGlaWaves) MLOP_GLA_C(N, 1); else MLOP_GLA_C(N, 2);   \
  } while (0)
  const int nkt = cdiv(a.dk, 16);
  if (nkt <= 1) MLOP_GLA(1);
  else if (nkt <= 2) MLOP_GLA(2);
  else if (nkt <= 4) MLOP_GLA(4);
  else if (nkt <= 6) MLOP_GLA(6);
  else if (nkt <= 8) MLOP_GLA(8);
  else if (nkt <= 12) MLOP_GLA(12);
  else MLOP_GLA(16);
#undef MLOP_GLA
#undef MLOP_GLA_C
}

}  // namespace mlop
