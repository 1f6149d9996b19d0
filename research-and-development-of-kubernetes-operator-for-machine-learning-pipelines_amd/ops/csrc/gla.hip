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
template <typename E, int VEC>
__global__ void __launch_bounds__(256) gla_rows_kernel(GlaArgs a, const int* __restrict__ rows) {
  extern __shared__ float sm[];
  __shared__ float scratch[16];
  const int s = rows[blockIdx.x], h = blockIdx.y, tid = threadIdx.x;
  const int dk = a.dk, dv = a.dv;
  float* a1 = sm;                  // [rank]
  float* dec = a1 + a.rank;        // [dk]
  float* q = dec + dk;             // [dk]
  float* k = q + dk;               // [dk]
  float* o = k + dk;               // [dv]
  float* red = o + dv;             // [256 * VEC]
  const int ql = a.q_len[s], ctx = a.ctx_len[s], qs = a.q_start[s];
  E* outp = reinterpret_cast<E*>(a.out);
  if (ctx < ql || s >= a.n_slots) {  // graph padding: attends to nothing, holds no state
    for (int t = 0; t < ql; ++t)
      for (int c = tid; c < dv; c += 256) st1(outp + ((size_t)(qs + t) * a.H + h) * dv + c, 0.f);
    return;
  }
  float* S = a.state + ((size_t)s * a.H + h) * dk * dv;
  const int nstrip = dv / VEC, per = min(nstrip, 256), RG = 256 / per;
  const int HK = a.H * dk, HV = a.H * dv;
  for (int t = 0; t < ql; ++t) {
    const E* row = reinterpret_cast<const E*>(a.proj) + (size_t)(qs + t) * a.ldp;
    const bool fresh = ctx - ql + t == 0;
    for (int i = tid; i < a.rank; i += 256) a1[i] = ld1(row + 2 * HK + 2 * HV + i);
    __syncthreads();
    for (int d = tid; d < dk; d += 256) {
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
#pragma unroll 8
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
      for (int c = tid; c < per * VEC; c += 256) {
        if (s0 * VEC + c < dv) {
          float x = 0.f;
          for (int g = 0; g < RG; ++g) x += red[g * per * VEC + c];
          o[s0 * VEC + c] = x;
        }
      }
      __syncthreads();
    }
    float ss = 0.f;
    for (int c = tid; c < dv; c += 256) ss = fmaf(o[c], o[c], ss);
    ss = block_sum(ss, scratch);
    const float inv = 1.f / sqrtf(ss / (float)dv + a.eps);
    const E* gp = row + 2 * HK + HV + h * dv;
    for (int c = tid; c < dv; c += 256)
      st1(outp + ((size_t)(qs + t) * a.H + h) * dv + c, o[c] * inv * a.norm_w[c] * silu_f(ld1(gp + c)));
  }
}

// logd[t, n] = log_sigmoid(z) / tau for 8 tokens per workgroup (A2 rows reused over them)
template <typename E>
__global__ void __launch_bounds__(256) gla_decay_kernel(GlaArgs a, float* __restrict__ logd, int T) {
  extern __shared__ float sm[];  // [8][rank]
  const int t0 = blockIdx.x * 8, n = min(8, T - t0), HK = a.H * a.dk, off = 2 * HK + 2 * a.H * a.dv;
  for (int i = threadIdx.x; i < n * a.rank; i += 256)
    sm[i] = ld1(reinterpret_cast<const E*>(a.proj) + (size_t)(t0 + i / a.rank) * a.ldp + off + i % a.rank);
  __syncthreads();
  for (int c = blockIdx.y * 256 + threadIdx.x; c < HK; c += gridDim.y * 256) {
    const E* w = reinterpret_cast<const E*>(a.a2) + (size_t)c * a.rank;
    const float b = a.a2_b[c];
    float z[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) z[j] = b;
    for (int i = 0; i < a.rank; ++i) {
      const float wi = ld1(w + i);
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (j < n) z[j] = fmaf(wi, sm[j * a.rank + i], z[j]);
    }
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (j < n) logd[(size_t)(t0 + j) * HK + c] = log_sigmoid(z[j]) * a.inv_tau;
  }
}

// One chunk of one head for a group of 16 NW value columns.  Thread d < dk owns key channel d in the
// elementwise part (its running decay over the block's 16 tokens); wave w owns 16 value columns in
// the products, the state [16 NKT, 16] in its accumulators.
//   OUT = false: the chunk's own contribution from a zero state -> cstate, total decay -> cdecay
//   OUT = true:  outputs from the chunk's starting state in cstate
template <typename E, int NKT, bool OUT>
__global__ void __launch_bounds__(512) gla_chunk_kernel(GlaArgs a, float* __restrict__ o32,
                                                        float* __restrict__ cstate, float* __restrict__ cdecay,
                                                        const float* __restrict__ logd,
                                                        const int* __restrict__ item_seq,
                                                        const int* __restrict__ item_t0, int chunk) {
  constexpr int DKP = 16 * NKT, LD = DKP + 4, LT = 20;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* KT = sm;                     // [DKP][LT]: k_j e^{b_16 - b_j}, token fastest
  float* En = KT + DKP * LT;          // [DKP]: e^{b_16}
  float* Qs = En + DKP;               // [16][LD]: q e^b
  float* Ks = Qs + 16 * LD;           // [16][LD]: k e^-b
  float* part = Ks + 16 * LD;         // [NW][256]
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, NW = blockDim.x >> 6;
  const int item = blockIdx.x, h = blockIdx.y;
  const int s = item_seq[item], t0 = item_t0[item];
  const int n = min(chunk, a.q_len[s] - t0), tok0 = a.q_start[s] + t0;
  const int dk = a.dk, dv = a.dv, HK = a.H * dk, HV = a.H * dv;
  const int l15 = lane & 15, g4 = lane >> 4;
  const int col = (blockIdx.z * NW + wid) * 16 + l15;
  const bool wave_cols = (blockIdx.z * NW + wid) * 16 < dv, col_ok = col < dv;
  const bool own = tid < DKP, own_ok = tid < dk;
  const E* proj = reinterpret_cast<const E*>(a.proj) + (size_t)tok0 * a.ldp;
  float* cst = cstate + ((size_t)item * a.H + h) * dk * dv;

  f32x4 S[NKT];
#pragma unroll
  for (int kt = 0; kt < NKT; ++kt) {
    S[kt] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (OUT && col_ok) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = 16 * kt + 4 * g4 + i;
        if (d < dk) S[kt][i] = cst[(size_t)d * dv + col];
      }
    }
  }
  float total = 0.f;
  for (int t = 0; t < n; t += 16) {
    const int nt = min(16, n - t);
    float b[16], kk[16], qq[16];
#pragma unroll
    for (int j = 0; j < 16; ++j) {
      const bool ok = own_ok && j < nt;
      b[j] = ok ? logd[(size_t)(tok0 + t + j) * HK + h * dk + tid] : 0.f;
      kk[j] = ok ? ld1(proj + (size_t)(t + j) * a.ldp + HK + h * dk + tid) : 0.f;
      if (OUT) qq[j] = ok ? ld1(proj + (size_t)(t + j) * a.ldp + h * dk + tid) * a.q_scale : 0.f;
    }
    float vv[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int j = 4 * g4 + i;
      vv[i] = (col_ok && j < nt) ? ld1(proj + (size_t)(t + j) * a.ldp + 2 * HK + h * dv + col) : 0.f;
    }
#pragma unroll
    for (int j = 1; j < 16; ++j) b[j] += b[j - 1];
    const float bn = b[15];
    total += bn;
    bool fast = true;
    if (OUT) fast = !__syncthreads_or(own && bn < kFastDecay);  // also: the last block's LDS reads are done
    else __syncthreads();
    auto put_kt = [&]() {
#pragma unroll
      for (int j = 0; j < 16; j += 4)
        *reinterpret_cast<f32x4*>(KT + tid * LT + j) =
            f32x4{kk[j] * expf(bn - b[j]), kk[j + 1] * expf(bn - b[j + 1]), kk[j + 2] * expf(bn - b[j + 2]),
                  kk[j + 3] * expf(bn - b[j + 3])};
    };
    if (own) {
      En[tid] = expf(bn);
      if (OUT) {
        if (fast) {
#pragma unroll
          for (int j = 0; j < 16; ++j) {
            const float e = expf(b[j]);
            Qs[j * LD + tid] = qq[j] * e;
            Ks[j * LD + tid] = kk[j] / e;
          }
        } else {
#pragma unroll
          for (int j = 0; j < 16; ++j) {
            Qs[j * LD + tid] = qq[j];
            Ks[j * LD + tid] = kk[j];
            KT[j * LD + tid] = b[j];  // (DKP * LT >= 16 * LD)
          }
        }
      }
      if (!OUT || fast) put_kt();
    }
    __syncthreads();
    f32x4 A = {0.f, 0.f, 0.f, 0.f};  // scores^T: row j = 4 g4 + i, column = token l15
    if (OUT) {
      int nsum = NW;
      if (fast) {
        f32x4 p = {0.f, 0.f, 0.f, 0.f};
        for (int kt = wid; kt < NKT; kt += NW) {
          const f32x4 x = *reinterpret_cast<const f32x4*>(Ks + l15 * LD + 16 * kt + 4 * g4);
          const f32x4 y = *reinterpret_cast<const f32x4*>(Qs + l15 * LD + 16 * kt + 4 * g4);
#pragma unroll
          for (int i = 0; i < 4; ++i) p = mfma4(x[i], y[i], p);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) part[wid * 256 + (4 * g4 + i) * 16 + l15] = p[i];
      } else {
        nsum = 1;
        if (tid < 256) {
          const int j = tid >> 4, tt = tid & 15;
          float x = 0.f;
          if (j <= tt)
            for (int d = 0; d < dk; ++d)
              x = fmaf(Qs[tt * LD + d] * Ks[j * LD + d], expf(KT[tt * LD + d] - KT[j * LD + d]), x);
          part[tid] = x;
        }
        __syncthreads();
        if (own) {
#pragma unroll
          for (int j = 0; j < 16; ++j) Qs[j * LD + tid] = qq[j] * expf(b[j]);
          put_kt();
        }
      }
      __syncthreads();
      for (int w = 0; w < nsum; ++w)
#pragma unroll
        for (int i = 0; i < 4; ++i) A[i] += part[w * 256 + (4 * g4 + i) * 16 + l15];
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (4 * g4 + i > l15) A[i] = 0.f;
    }
    if (wave_cols) {
      if (OUT) {
        f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < 4; ++i) o = mfma4(A[i], vv[i], o);
#pragma unroll
        for (int kt = 0; kt < NKT; ++kt) {
          const f32x4 y = *reinterpret_cast<const f32x4*>(Qs + l15 * LD + 16 * kt + 4 * g4);
#pragma unroll
          for (int i = 0; i < 4; ++i) o = mfma4(y[i], S[kt][i], o);
        }
        if (col_ok) {
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (4 * g4 + i < nt) o32[(size_t)(tok0 + t + 4 * g4 + i) * HV + h * dv + col] = o[i];
        }
      }
      if (!OUT || t + 16 < n) {
#pragma unroll
        for (int kt = 0; kt < NKT; ++kt) {
          const f32x4 e = *reinterpret_cast<const f32x4*>(En + 16 * kt + 4 * g4);
          const f32x4 x = *reinterpret_cast<const f32x4*>(KT + (16 * kt + l15) * LT + 4 * g4);
          S[kt] *= e;
#pragma unroll
          for (int i = 0; i < 4; ++i) S[kt] = mfma4(x[i], vv[i], S[kt]);
        }
      }
    }
  }
  if (!OUT) {
    if (col_ok) {
#pragma unroll
      for (int kt = 0; kt < NKT; ++kt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int d = 16 * kt + 4 * g4 + i;
          if (d < dk) cst[(size_t)d * dv + col] = S[kt][i];
        }
    }
    if (own_ok && blockIdx.z == 0) cdecay[((size_t)item * a.H + h) * dk + tid] = expf(total);
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

template <typename E>
static void run_rows(const GlaArgs& a, const int* rows, int n_rows, hipStream_t st) {
  const bool v4 = a.dv % 4 == 0;
  const size_t lds = (size_t)(a.rank + 3 * a.dk + a.dv + 256 * (v4 ? 4 : 1)) * 4;
  if (v4) gla_rows_kernel<E, 4><<<dim3(n_rows, a.H), 256, lds, st>>>(a, rows);
  else gla_rows_kernel<E, 1><<<dim3(n_rows, a.H), 256, lds, st>>>(a, rows);
}

void launch_gla_rows(const GlaArgs& a, bool f32, const int* rows, int n_rows, hipStream_t st) {
  if (n_rows == 0) return;
  if (f32) run_rows<float>(a, rows, n_rows, st);
  else run_rows<uint16_t>(a, rows, n_rows, st);
}

template <typename E, int NKT>
static void run_chunks(const GlaArgs& a, float* logd, float* o32, float* cstate, float* cdecay, int T,
                       const int* item_seq, const int* item_t0, int n_items, const int* crow_seq,
                       const int* crow_item0, int n_crows, int chunk, hipStream_t st) {
  const int HK = a.H * a.dk;
  gla_decay_kernel<E><<<dim3(cdiv(T, 8), std::min(8, cdiv(HK, 256))), 256, (size_t)8 * a.rank * 4, st>>>(a, logd, T);
  const int NW = a.dv <= 64 ? 4 : 8;
  const dim3 grid(n_items, a.H, cdiv(a.dv, 16 * NW));
  constexpr int DKP = 16 * NKT, LD = DKP + 4;
  const size_t lds1 = (size_t)(DKP * 20 + DKP) * 4, lds2 = lds1 + (size_t)(2 * 16 * LD + NW * 256) * 4;
  auto k1 = gla_chunk_kernel<E, NKT, false>;
  auto k2 = gla_chunk_kernel<E, NKT, true>;
  static bool attr = false;
  if (!attr) {
    (void)hipFuncSetAttribute((const void*)k2, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
    attr = true;
  }
  k1<<<grid, NW * 64, lds1, st>>>(a, nullptr, cstate, cdecay, logd, item_seq, item_t0, chunk);
  gla_scan_kernel<<<dim3(n_crows, a.H, cdiv(a.dk * a.dv, 256)), 256, 0, st>>>(a, cstate, cdecay, crow_seq, crow_item0,
                                                                              chunk);
  k2<<<grid, NW * 64, lds2, st>>>(a, o32, cstate, cdecay, logd, item_seq, item_t0, chunk);
  gla_gate_kernel<E><<<dim3(n_items, cdiv(chunk * a.H, 4)), 256, 0, st>>>(a, o32, item_seq, item_t0, chunk);
}

void launch_gla_chunks(const GlaArgs& a, bool f32, float* logd, float* o32, float* cstate, float* cdecay, int T,
                       const int* item_seq, const int* item_t0, int n_items, const int* crow_seq,
                       const int* crow_item0, int n_crows, int chunk, hipStream_t st) {
  if (n_items == 0) return;
#define MLOP_GLA(N)                                                                                             \
  do {                                                                                                          \
    if (f32) run_chunks<float, N>(a, logd, o32, cstate, cdecay, T, item_seq, item_t0, n_items, crow_seq,        \
                                  crow_item0, n_crows, chunk, st);                                              \
    else run_chunks<uint16_t, N>(a, logd, o32, cstate, cdecay, T, item_seq, item_t0, n_items, crow_seq,         \
                                 crow_item0, n_crows, chunk, st);                                               \
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
}

}  // namespace mlop
