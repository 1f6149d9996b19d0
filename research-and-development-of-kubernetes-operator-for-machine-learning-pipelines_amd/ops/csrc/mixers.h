// Launchers of the mixers and norms that hybrid decoders combine, beside hybrid.h's: fp32 residual
// with a norm behind the sublayer, gated group norm, short causal convolution, selective state space
// (SSD), generalized delta rule, latent attention, clamped gated feed-forward.  `f32` selects float
// operands; otherwise bf16.  Rows, items and crows are a step's lists (runtime/attn_meta.py):
// one-token rows, chunks of prompt portions, and the portions' sequences.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

namespace mlop {

// a step's sequences: per-row arrays and the lists of what runs
struct StepRows {
  const int *q_start, *q_len, *ctx_len;
  const int* rows;        // one-token rows
  int n_rows;
  const int *item_seq, *item_t0;  // chunks of prompt portions
  int n_items;
  const int *crow_seq, *crow_item0;  // portions: row and first item
  int n_crows, chunk;
  int n_slots;            // state slots (rows past them are graph padding)
};

// ---- residual (residual.hip)
struct ResidualArgs {
  float* x;               // [T, W]
  void* xn;               // [T, W] the next sublayer's input: norm_w * x / rms(x)
  const void* y;          // [T, W] sublayer output (null: the experts' alone)
  const void* rows;       // [R, W] or null: sublayer output gate[t] y[t] + sum_j row_w[t, j] rows[inv[t, j]] + self_w[t] self[t]
  const int* inv;         // [T, top], < 0: no row
  const float* gate;      // [T] or null
  const float* row_w;     // [T, top] or null: ones
  const void* self;       // [T, W] or null
  const float* self_w;    // [T]
  int top;
  const float* post_w;    // [W] or, post_one, one number: y is normed on its own, times this (null: added as it is)
  const float* norm_w;    // [W] or, norm_one, one number (null: xn = x)
  bool post_one, norm_one;
  const float *tanh_a, *tanh_b;  // one number, [W], or null: xn = norm_w * tanh(a x) + b instead
  const long* ids;        // [T]  (start: x = scale * table[id] + pos_table[pos])
  const void* table;      // [vocab, W]
  const void* pos_table;  // [n_pos, W] or null
  const int* pos;         // [T]
  long vocab, n_pos;
  float embed_scale, eps;
  int T, W;
  int n;                  // columns the mean square is over (the rest are zero)
  bool store;             // write x back
};
void launch_residual(const ResidualArgs& a, bool f32, hipStream_t st);
constexpr int kResidualMaxW = 16384;

// ---- gated group norm (residual.hip)
enum GateAct { kGateSilu = 0, kGateSigmoid = 1 };
struct GatedNormArgs {
  void* out;              // [T, n]
  const void* y;          // [T, n]
  const void* gate;       // [T, ldg], first n columns
  long ldg;
  const float* w;         // [n]
  float eps;
  int T, n, groups;       // equal parts of n, each divided by its own root mean square
  int act;                // GateAct
  bool gate_first;        // y act(gate) is normed; else the normed y is gated
};
void launch_gated_norm(const GatedNormArgs& a, bool f32, hipStream_t st);

// ---- clamped gated unit of interleaved gate / up columns (residual.hip)
// out[t, i] = g sigmoid(alpha g) (u + 1), g = min(gate, limit), u = clamp(up, -limit, limit); alpha 0: silu(gate) up
void launch_clamp_glu(void* out, const void* x, int T, int I, float alpha, float limit, bool f32, hipStream_t st);

// ---- short causal convolution + silu with its last inputs as state (short_conv.hip)
struct ConvArgs {
  void* out;              // [T, C]
  const void* x;          // [T, ldx], first C columns
  long ldx;
  const float* w;         // [C, taps], last column: the current token
  const float* b;         // [C] or null
  float* tail;            // [slots, taps - 1, C]: a sequence's last inputs, oldest first
  int C, taps;
};
void launch_short_conv(const ConvArgs& a, const StepRows& s, bool f32, hipStream_t st);
constexpr int kConvMaxTaps = 16;

// ---- selective state space (ssd.hip)
struct SsdArgs {
  void* y;                // [T, H * V]
  const void* xbc;        // [T, ldx]: x (H x V) | B (G x N) | C (G x N)
  long ldx;
  const void* dt;         // [T, ldt], first H columns (before bias and softplus)
  long ldt;
  const float *dt_bias, *a_neg, *d_skip;  // [H]: a_neg = -exp(A_log)
  float* state;           // [slots, H, N, V]
  int H, V, N, G;
};
// one-token rows in place; portions in blocks of 16 tokens over `ws` (ssd_ws_floats)
void launch_ssd(const SsdArgs& a, const StepRows& s, float* ws, bool f32, hipStream_t st);
long ssd_ws_floats(int n_items, int chunk, int H);
constexpr int kSsdMaxN = 256;    // state size of the prompt kernel (larger: token by token)

// ---- generalized delta rule (delta.hip)
struct DeltaArgs {
  void* o;                // [T, H * dv]
  const void* proj;       // [T, ldp]: r (H x dk) | k (H x dk) | v (H x dv) | a (H x dk) | w1 (rank) | ...
  long ldp;
  const void* w2;         // [H * dk, rank]
  const float *w0, *a_b;  // [H * dk]
  float* state;           // [slots, H, dk, dv]
  int H, dk, dv, rank;
  float decay_scale;      // log decay = -decay_scale * sigmoid(.)
  float unit_eps;         // in the key's unit norm
};
// one-token rows in place; portions in blocks of 16 tokens over `ws` (delta_ws_floats)
void launch_delta(const DeltaArgs& a, const StepRows& s, float* ws, bool f32, hipStream_t st);
long delta_ws_floats(int n_items, int chunk, int H, int dk);
bool delta_blocks_ok(int dk, float decay_scale);  // else portions run token by token, without workspace

// ---- latent attention (latent.hip; attention_hd.hip runs the softmax)
// c = w * l / rms(l) of latent rows l into the paged cache [NB, 1, BS, RP], with a rotated key part behind
// it; and / or the queries' latents, normed the same way, to rows of their own
struct LatentStoreArgs {
  void* cache;
  const void* l;          // [T, ldl], first R columns (null: no latents)
  long ldl;
  const float* w;         // [R]
  const int* slots;       // < 0: no cache write
  int R, RP;
  const void* k;          // [T, ldk], first n_rot columns: dims off .. off + n_rot of the row (null: none)
  long ldk;
  const float* table;     // [n_pos, n_rot]: cos of the pairs (2i, 2i + 1), then sin
  const int* pos;
  int n_rot, off, n_pos;
  void* q_out;            // [T, QP], columns past QR zero
  const void* q;          // [T, ldq], first QR columns (null: none)
  long ldq;
  const float* q_w;       // [QR]
  int QR, QP;
  float eps;
  int T;
};
void launch_latent_store(const LatentStoreArgs& a, bool f32, hipStream_t st);
// cached rows of every portion's keys, positions window_start .. context end, to out [rows, RP];
// row of position p of sequence s: xbase[s] + p; the `pad` rows behind them are zeroed
struct LatentGatherArgs {
  void* out;
  const void* cache;
  const int *bt, *xbase, *q_len, *ctx_len, *crow_seq;
  int bt_stride, n_crows, x_max, rows, pad, RP, BS, num_blocks, window;
};
void launch_latent_gather(const LatentGatherArgs& a, bool f32, hipStream_t st);
// per head h: out[i, h, n] = sum_k x[i, h, k] w[h, n, k] for the step's one-token tiles i
struct HeadMmArgs {
  void* out;
  const void* x;
  const void* w;          // [H, N, K]
  long ldx, hx, ldo, ho;  // row and head strides (elements)
  const int *tile_seq, *tile_q0, *q_start, *q_len;
  bool x_tok, out_tok;    // x / out rows: the tile's token (else the tile's index)
  const void* gate;       // [T, ldg]: out times sigmoid(gate[token, h * N + n]) (null: none)
  long ldg;
  int n_tiles, H, N, K;   // K a multiple of 64
  // columns N .. N + extra of out (table; null: none): x's dims x_off .. x_off + n_rot, turned by the
  // token's position, then zeros
  const float* table;     // [n_pos, n_rot]
  const int* pos;
  int extra, x_off, n_rot, n_pos;
};
void launch_head_mm(const HeadMmArgs& a, bool f32, hipStream_t st);

// first position of the keys a portion needs, on a page pair
__host__ __device__ inline int key_region_start(int start, int window) {
  const int lo = window > 0 ? start - window + 1 : 0;
  return lo > 0 ? lo & ~31 : 0;
}

}  // namespace mlop
