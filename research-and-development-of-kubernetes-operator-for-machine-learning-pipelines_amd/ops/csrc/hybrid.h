// Launchers of the hybrid-decoder kernels (hyper-connections, whole-projection or per-head query / key
// norm with partial rotary positions, paged attention of any head sizes with a softmax sink and an
// output gate, gated linear attention).  `f32` selects float operands; otherwise bf16.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

namespace mlop {

// ---- hyper-connections (hyper.hip)
struct HyperArgs {
  float* streams;        // [T, S, W]
  void* xn;              // [T, W] normed sublayer input
  const void* y;         // [T, W] sublayer output (null: streams start from the embedding)
  const long* ids;       // [T]     (start only)
  const void* table;     // [vocab, W] (start only)
  float embed_scale;
  long vocab;
  const float* mix;      // [S, S] (from, to)
  const float* w_out;    // [S]
  const float* w_in;     // [S] of the sublayer that reads next
  const float* norm_w;   // [W]
  float eps;
  int T, W, S;
  bool store;            // write the new streams back (off behind the last sublayer)
};
void launch_hyper(const HyperArgs& a, bool f32, hipStream_t st);
constexpr int kMaxStreams = 64;

// ---- query / key norm + rotary + value mixing + paged stores (qk_norm.hip)
struct QkNormArgs {
  void* q_out;           // [T, H, KP], dims past D zero
  void* k_cache;         // [NB, G, BS, KP]
  void* v_cache;         // [NB, G, BS, VP]
  const void* proj;      // [T, ldp]: q (H x D) | k (G x D) | v (G x V) | ...
  long ldp;
  const void* v_first;   // values to mix in, row stride ldf (null: none)
  long ldf;
  const float* lam;      // [1] share of v_first
  const float* q_w;      // [H * D] (null: no norm)
  const float* k_w;      // [G * D]
  float eps;
  const float* cos_sin;  // [max_pos, R]: cos of the R / 2 pairs, then sin
  int R;                 // rotated dims of a head (even; pairs 2i, 2i + 1)
  const int* pos;
  const int* slots;      // < 0: no cache write
  int T, H, G, D, V, KP, VP, BS;
};
void launch_qk_norm(const QkNormArgs& a, bool f32, hipStream_t st);

// ---- per-head query / key norm + rotary + paged stores (qk_norm.hip)
struct QkHeadNormArgs {
  void* q_out;           // [T, H, KP], dims past D zero
  void* k_cache;         // [NB, G, BS, KP]
  void* v_cache;         // [NB, G, BS, VP]
  const void *q, *k, *v; // [T, H x D], [T, G x D], [T, G x V]; v null: the values are k as given (V = D)
  long ldq, ldk, ldv;
  const float *q_w, *k_w;  // [D]: one weight for all heads, each divided by its own root mean square
  float eps;
  const float* cos_sin;  // [max_pos, R]: cos of the R / 2 pairs, then sin
  int R;                 // rotated dims of a head (even; pairs 2i, 2i + 1)
  const int* pos;
  const int* slots;      // < 0: no cache write
  int T, H, G, D, V, KP, VP, BS;
};
void launch_qk_head_norm(const QkHeadNormArgs& a, bool f32, hipStream_t st);

// ---- paged attention of any head sizes (attention_hd.hip)
struct AttnHdArgs {
  void* out;             // [T, H, V] (by_tile: [tiles, H, V]), rows out_row elements apart
  long out_row;
  const void* q;         // rows of KP per token (by_tile: per tile) and head
  long q_row, q_head;    // strides of q (elements)
  // keys and values, 16-token pages: row t of page p, head g at p * 16 * pitch + t * row + g * head.  Paged
  // caches [NB, G, 16, KP]; or dense rows (xbase: row of a sequence's position 0), where pitch = row
  const void* k_cache;
  const void* v_cache;
  long k_pitch, k_row, k_head, v_pitch, v_row, v_head;
  const int* xbase;      // dense: [sequences]; null: paged
  const int* bt;
  int bt_stride;
  const int *q_start, *q_len, *ctx_len;
  const float* sink;     // [H] or null
  const void* gate;      // [T, gate_stride] pre-sigmoid, or null
  long gate_stride;
  bool gate_elem;        // one gate per head and value element (H x V); else one per head
  bool gate_vec;         // element gates are read 4 at a time (aligned rows)
  bool by_tile;          // q and out rows are decode tiles, not tokens
  int window;            // a token sees itself and the window - 1 tokens before it (0: all)
  // prompt tiles: dims rot_lo .. rot_lo + n_rot of a query head turn by the token's position as they are
  // read (null: none); [n_pos, n_rot]: cos of the pairs (2i, 2i + 1), then sin
  const float* rot;
  int rot_lo, n_rot, n_pos;
  int H, G, D, V, KP, VP;
  float scale_log2;
  int num_blocks;
};
// one query token per tile, split over `nparts` ranges of `part_tokens` keys
void launch_paged_hd(const AttnHdArgs& a, bool f32, float* part_o, float* part_ml, int* sem, const int* tile_seq,
                     const int* tile_q0, int num_tiles, int part_tokens, int nparts, hipStream_t st);
// the same with keys and values the same latent rows (latent_decode.hip): by_tile, one head of KP = VP <=
// 576 elements, the first V of them values; partials per 16 heads
void launch_latent_decode(const AttnHdArgs& a, float* part_o, float* part_ml, const int* tile_seq, const int* tile_q0, int num_tiles, int part_tokens, int nparts, hipStream_t st);
inline bool latent_decode_ok(const AttnHdArgs& a, bool f32) {
  return !f32 && a.by_tile && a.G == 1 && a.k_cache == a.v_cache && a.KP == a.VP && a.V % 64 == 0 && a.KP <= 576;
}
// tiles of up to 128 query tokens of one head
void launch_flash_hd(const AttnHdArgs& a, bool f32, const int* tile_seq, const int* tile_q0, int num_tiles,
                     hipStream_t st);
constexpr int kHdTile = 128;      // query tokens of a flash tile
constexpr int kHdMaxDim = 256;    // head sizes of the MFMA kernels (larger ones take the plain kernel)
constexpr int kHdMaxV = 1024;     // value size of the plain kernel

// ---- gated linear attention (gla.hip)
struct GlaArgs {
  void* out;             // [T, H * dv] (normed and gated)
  const void* proj;      // [T, ldp]: q (H x dk) | k (H x dk) | v (H x dv) | g (H x dv) | a1 (rank)
  long ldp;
  const void* a2;        // [H * dk, rank]
  const float* a2_b;     // [H * dk]
  const float* norm_w;   // [dv]
  float* state;          // [slots, H, dk, dv]
  const int *q_start, *q_len, *ctx_len;
  int n_slots, H, dk, dv, rank;
  float inv_tau, q_scale, eps;
};
// every token of each listed row in turn (one-token rows; any sizes)
void launch_gla_rows(const GlaArgs& a, bool f32, const int* rows, int n_rows, hipStream_t st);
// chunks of `chunk` tokens in parallel; o32 [T, H, dv] (only if gla_chunks_need_o32), cstate
// [items, H, dk, dv], cdecay [items, H, dk] are scratch; crow_* list the sequences and their items
void launch_gla_chunks(const GlaArgs& a, bool f32, float* o32, float* cstate, float* cdecay, const int* item_seq,
                       const int* item_t0, int n_items, const int* crow_seq, const int* crow_item0, int n_crows,
                       int chunk, hipStream_t st);
bool gla_chunks_need_o32(int dv);
constexpr int kGlaMaxDk = 256;    // key size of the chunked kernel

// ---- elementwise (hyper.hip)
// an activation (launch.h kAct*) of columns n0 .. N, in place
void launch_act_columns(void* x, long rows, int N, int n0, int act, float a, float b, bool f32, hipStream_t st);
void launch_softcap(float* out, const void* x, long n, float cap, bool f32, hipStream_t st);

}  // namespace mlop
