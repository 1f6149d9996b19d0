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

template <typename E, int VEC, int BT, bool NT>
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
            ld_state<NT>(col + (size_t)d * V, x);
          }
          const float bd = bv[d], cd = cv[d];
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            x[e] = fmaf(de, x[e], bd * v[e]);
            acc[e] = fmaf(cd, x[e], acc[e]);
          }
          st_state<NT>(col + (size_t)d * V, x);
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

// Decays of a portion's blocks, per (block, head): running log2 decay b of the block's tokens, their step
// sizes dt (0 past the portion), e^{b_16 - b} dt, e^b.  Lane = token, 16 heads per workgroup.
constexpr int kSsdBlk = 16, kSsdDec = 4 * kSsdBlk;

template <typename E>
__global__ void __launch_bounds__(256) ssd_decay_kernel(SsdArgs a, StepRows r, float* __restrict__ ws) {
  const int nb = r.chunk / kSsdBlk, item = blockIdx.x / nb, h = blockIdx.y * 16 + (threadIdx.x >> 4), l15 = threadIdx.x & 15;
  const int s = r.item_seq[item], t = r.item_t0[item] + (int)blockIdx.x % nb * kSsdBlk + l15;
  const bool in = t < r.q_len[s];
  const int hc = min(h, a.H - 1);
  const size_t row = (size_t)r.q_start[s] + (in ? t : 0);
  const float raw = ld1(reinterpret_cast<const E*>(a.dt) + row * a.ldt + hc);
  const float dt = in ? softplus_f(raw + a.dt_bias[hc]) : 0.f;
  const float b = scan16(a.a_neg[hc] * kLog2E * dt), all = __shfl(b, 15, 16);
  if (h >= a.H) return;
  float* o = ws + ((size_t)blockIdx.x * a.H + h) * kSsdDec + l15;
  o[0] = b;
  o[16] = dt;
  o[32] = exp2_f(all - b) * dt;
  o[48] = exp2_f(b);
}

// State rows per wave: 32, in two accumulator tiles; tile k's row r is state row 8 (r >> 2) + 4 k + (r & 3), so
// that a lane's eight consecutive elements of B or C are the operands of both.
template <typename E, int NW, int NC, bool VEC>
__global__ void __launch_bounds__(64 * NW) ssd_walk_kernel(SsdArgs a, StepRows r, const float* __restrict__ ws,
                                                           int n_cols) {
  constexpr int M = 1 + NC;
  constexpr bool BF = sizeof(E) == 2;
  __shared__ __attribute__((aligned(16))) f32x4 part[2][NW][M][64];
  // units: head by head (a group's heads share B and C in one L2), then portion, then columns
  const int unit = xcd_unit(blockIdx.x, a.H * r.n_crows * n_cols);
  if (unit < 0) return;
  const int h = unit / (r.n_crows * n_cols), crow = unit / n_cols % r.n_crows, s = r.crow_seq[crow];
  const int lane = threadIdx.x & 63, wid = __builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6)), l15 = lane & 15, g4 = lane >> 4;
  const int N = a.N, V = a.V, HV = a.H * V, grp = h / (a.H / a.G);
  const int ql = r.q_len[s], ctx = r.ctx_len[s], q0 = r.q_start[s];
  if (s >= r.n_slots) return;
  const int col0 = unit % n_cols * 16 * NC, n0 = wid * 32;
  const float dsk = a.d_skip[h];
  float* st = a.state + ((size_t)s * a.H + h) * N * V;
  // this lane's state rows: 8 g4 + 4 k + i of the wave's (accumulators), and the one it feeds tile k (B^T)
  const int d8 = n0 + 8 * g4, dt_row = n0 + 8 * (l15 >> 2) + (l15 & 3);

  f32x4 S[2][NC];
#pragma unroll
  for (int k = 0; k < 2; ++k)
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      S[k][c] = f32x4{0.f, 0.f, 0.f, 0.f};
      const int col = col0 + 16 * c + l15;
      if (ctx != ql && col < V) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (d8 + 4 * k + i < N) S[k][c][i] = st[(size_t)(d8 + 4 * k + i) * V + col];
      }
    }

  // A block's operands as stored.  Offsets from the block's first row are per lane and fixed but for a
  // portion's last block, whose missing rows repeat its last one (their dt is zero); state rows past N
  // repeat the last ones (zeroed where they are used).
  struct Ops {
    Raw8<E> b, c;
    E bt[2][4], x[NC][4];
    float b1;
    f32x4 bj, dj, sj, eb;
  };
  const E* base = reinterpret_cast<const E*>(a.xbc) + (size_t)q0 * a.ldx;
  const uint32_t ldx = (uint32_t)a.ldx, ob = HV + grp * N, oc = HV + (a.G + grp) * N;
  const int dd = min(d8, VEC ? N - 8 : N - 1), last = N - 1 - dd;
  uint32_t row1, rows[4];
  auto offsets = [&](int n) {
    row1 = (uint32_t)min(l15, n - 1) * ldx;
#pragma unroll
    for (int i = 0; i < 4; ++i) rows[i] = (uint32_t)min(4 * g4 + i, n - 1) * ldx;
  };
  const float* dec = ws + ((size_t)r.crow_item0[crow] * (r.chunk / kSsdBlk) * a.H + h) * kSsdDec;
  const int t_last = (ql - 1) / kSsdBlk * kSsdBlk;
  // (never conditional: a branch around loads makes every later wait drain them all; past the last block
  // it repeats that one)
  auto fetch = [&](int t, Ops& o) {
    t = min(t, t_last);
    if (t + 16 > ql) offsets(ql - t);
    const E* p = base + (size_t)t * ldx;
    o.b.template load<VEC>(p + (row1 + ob + dd), last);
    o.c.template load<VEC>(p + (row1 + oc + dd), last);
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      const uint32_t dl = ob + min(dt_row + 4 * k, N - 1);
#pragma unroll
      for (int i = 0; i < 4; ++i) o.bt[k][i] = p[rows[i] + dl];
    }
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const uint32_t col = h * V + min(col0 + 16 * c + l15, V - 1);
#pragma unroll
      for (int i = 0; i < 4; ++i) o.x[c][i] = p[rows[i] + col];
    }
    const float* d = dec + (size_t)(t / kSsdBlk) * a.H * kSsdDec;
    o.b1 = d[l15];
    o.bj = *reinterpret_cast<const f32x4*>(d + 4 * g4);
    o.dj = *reinterpret_cast<const f32x4*>(d + 16 + 4 * g4);
    o.sj = *reinterpret_cast<const f32x4*>(d + 32 + 4 * g4);
    o.eb = *reinterpret_cast<const f32x4*>(d + 48 + 4 * g4);
  };
  offsets(16);
  auto step = [&](int blk, const Ops& cur, Ops& fill) {
    const int t = blk * kSsdBlk, buf = blk & 1;
    fetch(t + 2 * kSsdBlk, fill);
    f32x4 sc = {0.f, 0.f, 0.f, 0.f};  // B C^T: row j = 4 g4 + i, column = token l15
    f32x4 yp[NC];
#pragma unroll
    for (int c = 0; c < NC; ++c) yp[c] = f32x4{0.f, 0.f, 0.f, 0.f};
    if constexpr (BF) {
      u32x4 b = cur.b.v;
      if (n0 + 32 > N) {  // (one side zero is enough)
#pragma unroll
        for (int e = 0; e < 4; ++e)
          b[e] = d8 + 2 * e + 1 < N ? b[e] : d8 + 2 * e < N ? b[e] & 0xffffu : 0u;
      }
      sc = mfma16(__builtin_bit_cast(bf16x8, b), __builtin_bit_cast(bf16x8, cur.c.v), sc);
    }
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      const f32x4 ck = cur.c.f(k);
      if constexpr (!BF) {
        f32x4 bk = cur.b.f(k);
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (d8 + 4 * k + i >= N) bk[i] = 0.f;
        sc = mfma_f32x16(bk, ck, sc);
      }
#pragma unroll
      for (int c = 0; c < NC; ++c) yp[c] = mfma_f32x16(ck, S[k][c], yp[c]);
    }
    part[buf][wid][0][lane] = sc;
#pragma unroll
    for (int c = 0; c < NC; ++c) part[buf][wid][1 + c][lane] = yp[c];
    // the state behind the block
    const float eall = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(cur.eb[3]), 63));
    f32x4 x[NC];
    u32x2 btp[2];
    if constexpr (BF) {
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        btp[k] = u32x2{(uint32_t)cur.bt[k][0] | (uint32_t)cur.bt[k][1] << 16, (uint32_t)cur.bt[k][2] | (uint32_t)cur.bt[k][3] << 16};
        if (dt_row + 4 * k >= N) btp[k] = u32x2{0u, 0u};
      }
    }
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      x[c] = f32x4{ld1(&cur.x[c][0]), ld1(&cur.x[c][1]), ld1(&cur.x[c][2]), ld1(&cur.x[c][3])};
      const f32x4 xs = x[c] * cur.sj;
#pragma unroll
      for (int k = 0; k < 2; ++k) S[k][c] *= eall;
      if constexpr (BF) {
        u32x2 xp[3];
        split3(xs, xp);
#pragma unroll
        for (int p = 2; p >= 0; --p)
#pragma unroll
          for (int k = 0; k < 2; ++k) S[k][c] = mfma_bf16x16(btp[k], xp[p], S[k][c]);
      } else {
#pragma unroll
        for (int k = 0; k < 2; ++k) {
          f32x4 bt;
#pragma unroll
          for (int i = 0; i < 4; ++i) bt[i] = dt_row + 4 * k < N ? ld1(&cur.bt[k][i]) : 0.f;
          S[k][c] = mfma_f32x16(bt, xs, S[k][c]);
        }
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
        G[i] = 4 * g4 + i <= l15 ? G[i] * cur.dj[i] * exp2_f(cur.b1 - cur.bj[i]) : 0.f;
        y[i] = fmaf(y[i], cur.eb[i], dsk * x[c][i]);
      }
      y = mfma_f32x16(G, x[c], y);
      const int col = col0 + 16 * c + l15;
      E* out = reinterpret_cast<E*>(a.y) + (size_t)(q0 + t) * HV + h * V + col;
      if (col < V) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (t + 4 * g4 + i < ql) st1(out + (size_t)(4 * g4 + i) * HV, y[i]);
      }
    }
  };
  Ops o0, o1, o2;
  fetch(0, o0);
  fetch(kSsdBlk, o1);
  const int nblk = cdiv(ql, kSsdBlk);
  int blk = 0;
  for (; blk + 3 <= nblk; blk += 3) {
    step(blk, o0, o2);
    step(blk + 1, o1, o0);
    step(blk + 2, o2, o1);
  }
  if (blk < nblk) step(blk, o0, o2);
  if (blk + 1 < nblk) step(blk + 1, o1, o0);
#pragma unroll
  for (int k = 0; k < 2; ++k)
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = d8 + 4 * k + i, col = col0 + 16 * c + l15;
        if (d < N && col < V) st[(size_t)d * V + col] = S[k][c][i];
      }
}

template <typename E, int BT>
static void ssd_rows_t(const SsdArgs& a, const StepRows& s, const int* rows, int n, hipStream_t st) {
  const bool v4 = a.V % 4 == 0;
  const size_t lds = (size_t)(2 * a.N + BT * (v4 ? 4 : 1)) * 4;
  if (v4 && (size_t)n * a.H * a.N * a.V * 4 >= kStreamBytes) ssd_rows_kernel<E, 4, BT, true><<<dim3(n, a.H), BT, lds, st>>>(a, s, rows);
  else if (v4) ssd_rows_kernel<E, 4, BT, false><<<dim3(n, a.H), BT, lds, st>>>(a, s, rows);
  else ssd_rows_kernel<E, 1, BT, false><<<dim3(n, a.H), BT, lds, st>>>(a, s, rows);
}

template <typename E>
static void ssd_rows(const SsdArgs& a, const StepRows& s, const int* rows, int n, hipStream_t st) {
  if (n == 0) return;
  // few (row, head) pairs: a whole CU's threads on each, so that its state is in flight at once
  if (n * a.H <= 256 && (long)a.N * a.V >= 8192) ssd_rows_t<E, 1024>(a, s, rows, n, st);
  else ssd_rows_t<E, 256>(a, s, rows, n, st);
}

template <typename E>
static void ssd_all(const SsdArgs& a, const StepRows& s, float* ws, hipStream_t st) {
  ssd_rows<E>(a, s, s.rows, s.n_rows, st);
  if (s.n_crows == 0) return;
  if (a.N > kSsdMaxN) return ssd_rows<E>(a, s, s.crow_seq, s.n_crows, st);
  ssd_decay_kernel<E><<<dim3(s.n_items * (s.chunk / kSsdBlk), cdiv(a.H, 16)), 256, 0, st>>>(a, s, ws);
  const bool vec = a.N % 8 == 0 && a.H * a.V % 8 == 0 && a.ldx % 8 == 0;
  const int c1 = cdiv(a.V, 16), c2 = cdiv(a.V, 32), u1 = a.H * s.n_crows * c1, u2 = a.H * s.n_crows * c2;
  const bool wide = a.V > 16 && u2 >= 256;  // (32 columns share the scores; 16 fill the chip sooner)
#define MLOP_WALK(NW)                                                                                        \
  do {                                                                                                       \
    if (!vec) ssd_walk_kernel<E, NW, 1, false><<<xcd_grid(u1), 64 * NW, 0, st>>>(a, s, ws, c1);              \
    else if (wide) ssd_walk_kernel<E, NW, 2, true><<<xcd_grid(u2), 64 * NW, 0, st>>>(a, s, ws, c2);          \
    else ssd_walk_kernel<E, NW, 1, true><<<xcd_grid(u1), 64 * NW, 0, st>>>(a, s, ws, c1);                    \
  } while (0)
  if (a.N <= 32) MLOP_WALK(1);
  else if (a.N <= 64) MLOP_WALK(2);
  else if (a.N <= 128) MLOP_WALK(4);
  else MLOP_WALK(8);
#undef MLOP_WALK
}

long ssd_ws_floats(int n_items, int chunk, int H) { return (long)n_items * (chunk / kSsdBlk) * H * kSsdDec; }

void launch_ssd(const SsdArgs& a, const StepRows& s, float* ws, bool f32, hipStream_t st) {
  if (f32) ssd_all<float>(a, s, ws, st);
  else ssd_all<uint16_t>(a, s, ws, st);
}

}  // namespace mlop
