// Selective state space (Mamba-2's state-space duality): per head a matrix state S [N, V] in fp32,
//
//   S_t = exp(A dt_t) S_{t-1} + dt_t B_t x_t^T,      y_t = S_t^T C_t + D x_t,      dt = softplus(raw + bias)
//
// with one scalar decay per head and token, and B, C shared by the heads of a group.  Everything of the
// recurrence is fp32 (x, B, C arrive in the model dtype); the matrix products use the fp32 MFMA.
//
//   ssd_rows_kernel   one-token rows: a workgroup per (row, head) streams the state once (HBM-bound);
//   ssd_walk_kernel   prompt portions: a workgroup per (sequence, head, 16 NC columns of V) walks the
//                     portion in blocks of 16 tokens with the state in its accumulators, its 4 waves
//                     splitting N.  With b_t the running sum of A dt inside a block,
//                       y_t = e^{b_t} C_t S + sum_{j <= t} e^{b_t - b_j} dt_j (C_t . B_j) x_j + D x_t
//                       S  <- e^{b_16} S + sum_j e^{b_16 - b_j} dt_j B_j x_j^T
//                     every exponent is <= 0.  The waves' partial C S and C B^T meet in LDS, one barrier
//                     per block.
//
// A sequence's first token starts from the zero state whatever its slot holds.
#include "mixers.h"
#include "recur.h"

namespace mlop {

template <typename E, int VEC, int BT>
__global__ void __launch_bounds__(BT) ssd_rows_kernel(SsdArgs a, StepRows r, const int* __restrict__ rows) {
  extern __shared__ float sm[];
  const int s = rows[blockIdx.x], h = blockIdx.y, tid = threadIdx.x;
  const int N = a.N, V = a.V;
  float* cv = sm;                  // [N] C
  float* bv = cv + N;              // [N] dt B
  float* red = bv + N;             // [BT * VEC]
  const int ql = r.q_len[s], ctx = r.ctx_len[s], q0 = r.q_start[s];
  const int HV = a.H * V, grp = h / (a.H / a.G);
  E* yp = reinterpret_cast<E*>(a.y) + (size_t)q0 * HV + h * V;
  if (ctx < ql || s >= r.n_slots) {  // graph padding: holds no state
    for (int t = 0; t < ql; ++t)
      for (int c = tid; c < V; c += BT) st1(yp + (size_t)t * HV + c, 0.f);
    return;
  }
  float* S = a.state + ((size_t)s * a.H + h) * N * V;
  const int nstrip = V / VEC, per = min(nstrip, BT), RG = BT / per;
  for (int t = 0; t < ql; ++t) {
    const E* row = reinterpret_cast<const E*>(a.xbc) + (size_t)(q0 + t) * a.ldx;
    const bool fresh = ctx - ql + t == 0;
    const float dt = softplus_f(ld1(reinterpret_cast<const E*>(a.dt) + (size_t)(q0 + t) * a.ldt + h) + a.dt_bias[h]);
    const float de = expf(a.a_neg[h] * dt), dsk = a.d_skip[h];
    for (int d = tid; d < N; d += BT) {
      bv[d] = dt * ld1(row + HV + grp * N + d);
      cv[d] = ld1(row + HV + (a.G + grp) * N + d);
    }
    __syncthreads();
    for (int s0 = 0; s0 < nstrip; s0 += per) {
      const int strip = s0 + tid % per, rg = tid / per;
      float acc[VEC], v[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) acc[e] = 0.f;
      if (rg < RG && strip < nstrip) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] = ld1(row + h * V + strip * VEC + e);
        float* col = S + strip * VEC;
#pragma unroll BT >= 1024 ? 4 : 8
        for (int d = rg; d < N; d += RG) {
          float x[VEC];
          if (fresh) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) x[e] = 0.f;
          } else {
            ldn<VEC>(col + (size_t)d * V, x);
          }
          const float bd = bv[d], cd = cv[d];
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            x[e] = fmaf(de, x[e], bd * v[e]);
            acc[e] = fmaf(cd, x[e], acc[e]);
          }
          stn<VEC>(col + (size_t)d * V, x);
        }
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) red[tid * VEC + e] = acc[e];
      __syncthreads();
      for (int c = tid; c < per * VEC; c += BT) {
        if (s0 * VEC + c < V) {
          float x = dsk * ld1(row + h * V + s0 * VEC + c);
          for (int g = 0; g < RG; ++g) x += red[g * per * VEC + c];
          st1(yp + (size_t)t * HV + s0 * VEC + c, x);
        }
      }
      __syncthreads();
    }
  }
}

template <typename E, int KT, int NC>
__global__ void __launch_bounds__(256) ssd_walk_kernel(SsdArgs a, StepRows r) {
  constexpr int NW = 4, M = 1 + NC;
  __shared__ __attribute__((aligned(16))) f32x4 part[2][NW][M][64];
  const int crow = blockIdx.x / a.H, h = blockIdx.x % a.H, s = r.crow_seq[crow];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, l15 = lane & 15, g4 = lane >> 4;
  const int N = a.N, V = a.V, HV = a.H * V, grp = h / (a.H / a.G);
  const int ql = r.q_len[s], ctx = r.ctx_len[s], q0 = r.q_start[s];
  if (s >= r.n_slots) return;
  const int col0 = (int)blockIdx.y * 16 * NC, n0 = wid * KT * 16;
  const E* xr = reinterpret_cast<const E*>(a.xbc) + (size_t)q0 * a.ldx;
  const E* xp = xr + h * V;
  const E* bp = xr + HV + grp * N;
  const E* cp = xr + HV + (a.G + grp) * N;
  const E* dtp = reinterpret_cast<const E*>(a.dt) + (size_t)q0 * a.ldt + h;
  const bool vec = HV % 4 == 0 && N % 4 == 0 && a.ldx % 4 == 0;
  const float a2 = a.a_neg[h] * kLog2E, bias = a.dt_bias[h], dsk = a.d_skip[h];
  float* st = a.state + ((size_t)s * a.H + h) * N * V;

  f32x4 S[KT][NC];
#pragma unroll
  for (int k = 0; k < KT; ++k)
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      S[k][c] = f32x4{0.f, 0.f, 0.f, 0.f};
      const int col = col0 + 16 * c + l15;
      if (ctx != ql && col < V) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int d = n0 + 16 * k + 4 * g4 + i;
          if (d < N) S[k][c][i] = st[(size_t)d * V + col];
        }
      }
    }

  // a block's operands; rows past the portion repeat its last one (their dt is zero)
  struct Ops {
    f32x4 b[KT], c[KT], bt[KT], x[NC];
    float dt;
  };
  auto fetch = [&](int t, Ops& o) {
    const E* br = bp + (size_t)min(t + l15, ql - 1) * a.ldx;
    const E* cr = cp + (size_t)min(t + l15, ql - 1) * a.ldx;
#pragma unroll
    for (int k = 0; k < KT; ++k) {
      const int d = n0 + 16 * k + 4 * g4, dd = min(d, N - 1);
      o.b[k] = ld4m(br + dd, N - d, vec);
      o.c[k] = ld4m(cr + dd, N - d, vec);
      const int dl = n0 + 16 * k + l15;
#pragma unroll
      for (int i = 0; i < 4; ++i)
        o.bt[k][i] = dl < N ? ld1(bp + (size_t)min(t + 4 * g4 + i, ql - 1) * a.ldx + dl) : 0.f;
    }
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int col = min(col0 + 16 * c + l15, V - 1);
#pragma unroll
      for (int i = 0; i < 4; ++i) o.x[c][i] = ld1(xp + (size_t)min(t + 4 * g4 + i, ql - 1) * a.ldx + col);
    }
    o.dt = ld1(dtp + (size_t)min(t + l15, ql - 1) * a.ldt);
  };
  Ops cur, nxt;
  fetch(0, cur);
  for (int t = 0, blk = 0; t < ql; t += 16, ++blk) {
    if (t + 16 < ql) fetch(t + 16, nxt);
    const int buf = blk & 1;
    // dt of token l15, running log2 decay over the block
    const float dt = t + l15 < ql ? softplus_f(cur.dt + bias) : 0.f;
    float b = a2 * dt;
#pragma unroll
    for (int d = 1; d < 16; d <<= 1) {
      const float up = __shfl_up(b, d, 16);
      if (l15 >= d) b += up;
    }
    const float ball = __shfl(b, 15);
    float bj[4], dj[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      bj[i] = __shfl(b, 4 * g4 + i);
      dj[i] = __shfl(dt, 4 * g4 + i);
    }
    f32x4 sc = {0.f, 0.f, 0.f, 0.f};  // row j = 4 g4 + i, column = token l15
    f32x4 yp[NC];
#pragma unroll
    for (int c = 0; c < NC; ++c) yp[c] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < KT; ++k) {
      sc = mfma_f32x16(cur.b[k], cur.c[k], sc);
#pragma unroll
      for (int c = 0; c < NC; ++c) yp[c] = mfma_f32x16(cur.c[k], S[k][c], yp[c]);
    }
    part[buf][wid][0][lane] = sc;
#pragma unroll
    for (int c = 0; c < NC; ++c) part[buf][wid][1 + c][lane] = yp[c];
    // the state behind the block
    const float eall = exp2_f(ball);
    float sj[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) sj[i] = exp2_f(ball - bj[i]) * dj[i];
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      f32x4 xs;
#pragma unroll
      for (int i = 0; i < 4; ++i) xs[i] = cur.x[c][i] * sj[i];
#pragma unroll
      for (int k = 0; k < KT; ++k) {
        S[k][c] *= eall;
        S[k][c] = mfma_f32x16(cur.bt[k], xs, S[k][c]);
      }
    }
    lds_sync();
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      if (((blk * NC + c) & (NW - 1)) != wid) continue;  // the waves take the finishing in turn
      f32x4 G = {0.f, 0.f, 0.f, 0.f}, y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int w = 0; w < NW; ++w) {
        G += part[buf][w][0][lane];
        y += part[buf][w][1 + c][lane];
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        G[i] = 4 * g4 + i <= l15 ? G[i] * dj[i] * exp2_f(b - bj[i]) : 0.f;
        y[i] = fmaf(y[i], exp2_f(bj[i]), dsk * cur.x[c][i]);
      }
      y = mfma_f32x16(G, cur.x[c], y);
      const int col = col0 + 16 * c + l15;
      E* out = reinterpret_cast<E*>(a.y) + (size_t)(q0 + t) * HV + h * V + col;
      if (col < V) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (t + 4 * g4 + i < ql) st1(out + (size_t)(4 * g4 + i) * HV, y[i]);
      }
    }
    cur = nxt;
  }
#pragma unroll
  for (int k = 0; k < KT; ++k)
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = n0 + 16 * k + 4 * g4 + i, col = col0 + 16 * c + l15;
        if (d < N && col < V) st[(size_t)d * V + col] = S[k][c][i];
      }
}

template <typename E, int BT>
static void ssd_rows_t(const SsdArgs& a, const StepRows& s, const int* rows, int n, hipStream_t st) {
  const bool v4 = a.V % 4 == 0;
  const size_t lds = (size_t)(2 * a.N + BT * (v4 ? 4 : 1)) * 4;
  if (v4) ssd_rows_kernel<E, 4, BT><<<dim3(n, a.H), BT, lds, st>>>(a, s, rows);
  else ssd_rows_kernel<E, 1, BT><<<dim3(n, a.H), BT, lds, st>>>(a, s, rows);
}

template <typename E>
static void ssd_rows(const SsdArgs& a, const StepRows& s, const int* rows, int n, hipStream_t st) {
  if (n == 0) return;
  // few (row, head) pairs: a whole CU's threads on each, so that its state is in flight at once
  if (n * a.H <= 256 && (long)a.N * a.V >= 8192) ssd_rows_t<E, 1024>(a, s, rows, n, st);
  else ssd_rows_t<E, 256>(a, s, rows, n, st);
}

template <typename E>
static void ssd_all(const SsdArgs& a, const StepRows& s, hipStream_t st) {
  ssd_rows<E>(a, s, s.rows, s.n_rows, st);
  if (s.n_crows == 0) return;
  if (a.N > kSsdMaxN) return ssd_rows<E>(a, s, s.crow_seq, s.n_crows, st);
  const bool wide = a.V > 16 && s.n_crows * a.H * cdiv(a.V, 32) >= 256;
#define MLOP_WALK(KT)                                                                                             \
  do {                                                                                                            \
    if (wide) ssd_walk_kernel<E, KT, 2><<<dim3(s.n_crows * a.H, cdiv(a.V, 32)), 256, 0, st>>>(a, s);              \
    else ssd_walk_kernel<E, KT, 1><<<dim3(s.n_crows * a.H, cdiv(a.V, 16)), 256, 0, st>>>(a, s);                   \
  } while (0)
  if (a.N <= 64) MLOP_WALK(1);
  else if (a.N <= 128) MLOP_WALK(2);
  else MLOP_WALK(4);
#undef MLOP_WALK
}

void launch_ssd(const SsdArgs& a, const StepRows& s, bool f32, hipStream_t st) {
  if (f32) ssd_all<float>(a, s, st);
  else ssd_all<uint16_t>(a, s, st);
}

}  // namespace mlop
