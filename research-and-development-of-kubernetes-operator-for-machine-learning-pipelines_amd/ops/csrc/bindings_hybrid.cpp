// torch.ops.mlop.* registrations of the hybrid-decoder kernels (hybrid.h): hyper-connections,
// query / key norm + rotary + paged stores, paged attention of any head sizes, gated linear
// attention.  As in bindings.cpp every op checks types and shapes on the host before it launches.
#include <cmath>

#include "bind_util.h"
#include "hybrid.h"
#include "launch.h"

namespace {

void hyper_common(mlop::HyperArgs& a, const Tensor& xn, const Tensor& streams, const Tensor& w_in, const Tensor& norm_w,
                  double eps) {
  TORCH_CHECK(streams.dim() == 3 && streams.is_contiguous() && streams.scalar_type() == at::kFloat && streams.is_cuda(),
              "streams must be [T, S, W] fp32");
  a.T = (int)streams.size(0);
  a.S = (int)streams.size(1);
  a.W = (int)streams.size(2);
  TORCH_CHECK(a.S >= 1 && a.S <= mlop::kMaxStreams, "1 .. ", mlop::kMaxStreams, " streams");
  TORCH_CHECK(a.W >= 1 && a.W <= 15360, "row width 1 .. 15360");
  TORCH_CHECK(xn.is_contiguous() && xn.numel() == (int64_t)a.T * a.W, "xn must be [T, W]");
  a.streams = streams.data_ptr<float>();
  a.xn = xn.data_ptr();
  a.w_in = f32_of(w_in, a.S, "w_in");
  a.norm_w = f32_of(norm_w, a.W, "norm_w");
  a.eps = (float)eps;
  aligned16(xn, "xn");
  aligned16(streams, "streams");
  aligned16(norm_w, "norm_w");
}

void hyper_begin(Tensor xn, Tensor streams, Tensor ids, Tensor table, double scale, Tensor w_in, Tensor norm_w, double eps) {
  mlop::HyperArgs a{};
  const bool f32 = model_f32(table, "table");
  like(xn, table, "xn");
  hyper_common(a, xn, streams, w_in, norm_w, eps);
  TORCH_CHECK(ids.is_cuda() && ids.scalar_type() == at::kLong && ids.is_contiguous() && ids.numel() == a.T, "ids int64 [T]");
  TORCH_CHECK(table.dim() == 2 && table.is_contiguous() && table.size(1) == a.W, "table must be [vocab, W]");
  aligned16(table, "table");
  a.ids = ids.data_ptr<int64_t>();
  a.table = table.data_ptr();
  a.vocab = table.size(0);
  a.embed_scale = (float)scale;
  a.store = true;
  c10::DeviceGuard g(table.device());
  mlop::launch_hyper(a, f32, cur());
}

void hyper_step(Tensor xn, Tensor streams, Tensor y, Tensor mix, Tensor w_out, Tensor w_in, Tensor norm_w, double eps,
                bool store) {
  mlop::HyperArgs a{};
  const bool f32 = model_f32(y, "y");
  like(xn, y, "xn");
  hyper_common(a, xn, streams, w_in, norm_w, eps);
  TORCH_CHECK(y.is_contiguous() && y.numel() == (int64_t)a.T * a.W, "y must be [T, W]");
  aligned16(y, "y");
  a.y = y.data_ptr();
  a.mix = f32_of(mix, (int64_t)a.S * a.S, "mix");
  a.w_out = f32_of(w_out, a.S, "w_out");
  a.store = store;
  c10::DeviceGuard g(y.device());
  mlop::launch_hyper(a, f32, cur());
}

void act_columns(Tensor x, int64_t n0, int64_t epi, double a, double b) {
  const bool f32 = model_f32(x, "x");
  TORCH_CHECK(x.is_contiguous() && x.dim() >= 1, "x must be contiguous");
  const int64_t N = x.size(-1);
  TORCH_CHECK(n0 >= 0 && n0 <= N && N < (1 << 30) && mlop::epi_act((int)epi), "columns, activation");
  aligned16(x, "x");
  c10::DeviceGuard g(x.device());
  mlop::launch_act_columns(x.data_ptr(), N ? x.numel() / N : 0, (int)N, (int)n0, mlop::epi_act((int)epi), (float)a, (float)b, f32,
                           cur());
}

void softcap(Tensor out, Tensor x, double cap) {
  const bool f32 = model_f32(x, "x");
  TORCH_CHECK(x.is_contiguous() && cap > 0, "x must be contiguous, cap > 0");
  f32_of(out, x.numel(), "out");
  aligned16(x, "x");
  c10::DeviceGuard g(x.device());
  mlop::launch_softcap(out.data_ptr<float>(), x.data_ptr(), x.numel(), (float)cap, f32, cur());
}

void qk_norm_rope(Tensor q_out, Tensor k_cache, Tensor v_cache, Tensor proj, int64_t D, int64_t V, OptT q_w, OptT k_w,
                  double eps, Tensor cos_sin, Tensor pos, Tensor slots, OptT v_first, OptT lam) {
  mlop::QkNormArgs a{};
  const bool f32 = model_f32(proj, "proj");
  like(q_out, proj, "q_out");
  like(k_cache, proj, "k_cache");
  like(v_cache, proj, "v_cache");
  TORCH_CHECK(q_out.dim() == 3 && q_out.is_contiguous() && k_cache.dim() == 4 && k_cache.is_contiguous() &&
                  v_cache.dim() == 4 && v_cache.is_contiguous() && proj.dim() == 2,
              "qk_norm_rope ranks");
  a.T = (int)q_out.size(0);
  a.H = (int)q_out.size(1);
  a.KP = (int)q_out.size(2);
  a.G = (int)k_cache.size(1);
  a.BS = (int)k_cache.size(2);
  a.VP = (int)v_cache.size(3);
  a.D = (int)D;
  a.V = (int)V;
  TORCH_CHECK(k_cache.size(3) == a.KP && v_cache.size(0) == k_cache.size(0) && v_cache.size(1) == a.G &&
                  v_cache.size(2) == a.BS,
              "caches must be [NB, G, BS, KP] and [NB, G, BS, VP]");
  TORCH_CHECK(D >= 2 && D % 2 == 0 && D <= a.KP && V >= 1 && V <= a.VP && a.KP % 8 == 0, "head sizes");
  TORCH_CHECK(a.H % a.G == 0, "query heads must be a multiple of kv heads");
  TORCH_CHECK(proj.size(0) == a.T && proj.size(1) >= a.H * D + a.G * (D + V), "proj is too narrow");
  a.ldp = proj.stride(0);
  aligned16(proj, "proj");
  aligned16(q_out, "q_out");
  aligned16(k_cache, "k_cache");
  TORCH_CHECK(q_w.has_value() == k_w.has_value(), "q and k norms come together");
  if (q_w) {
    a.q_w = f32_of(*q_w, a.H * D, "q_w");
    a.k_w = f32_of(*k_w, a.G * D, "k_w");
    aligned16(*q_w, "q_w");
    aligned16(*k_w, "k_w");
  }
  a.eps = (float)eps;
  TORCH_CHECK(cos_sin.dim() == 2 && cos_sin.is_cuda() && cos_sin.scalar_type() == at::kFloat && cos_sin.is_contiguous(),
              "cos_sin must be [max_pos, R] fp32");
  a.R = (int)cos_sin.size(1);
  TORCH_CHECK(a.R % 2 == 0 && a.R <= D, "rotated dims must be even and at most the head size");
  a.cos_sin = cos_sin.data_ptr<float>();
  a.pos = i32_of(pos, "pos");
  a.slots = i32_of(slots, "slots");
  TORCH_CHECK(pos.numel() == a.T && slots.numel() == a.T, "pos / slots length");
  if (v_first) {
    like(*v_first, proj, "v_first");
    TORCH_CHECK(v_first->dim() == 2 && v_first->size(0) == a.T && v_first->size(1) == a.G * V && lam.has_value(),
                "v_first must be [T, G * V], with lam");
    a.v_first = v_first->data_ptr();
    a.ldf = v_first->stride(0);
    a.lam = f32_of(*lam, 1, "lam");
  }
  a.q_out = q_out.data_ptr();
  a.k_cache = k_cache.data_ptr();
  a.v_cache = v_cache.data_ptr();
  a.proj = proj.data_ptr();
  c10::DeviceGuard g(proj.device());
  mlop::launch_qk_norm(a, f32, cur());
}

void qk_head_norm(Tensor q_out, Tensor k_cache, Tensor v_cache, Tensor q, Tensor k, OptT v, int64_t D, int64_t V, Tensor q_w,
                  Tensor k_w, double eps, Tensor cos_sin, Tensor pos, Tensor slots) {
  mlop::QkHeadNormArgs a{};
  const bool f32 = model_f32(q, "q");
  like(k, q, "k");
  like(q_out, q, "q_out");
  like(k_cache, q, "k_cache");
  like(v_cache, q, "v_cache");
  TORCH_CHECK(q_out.dim() == 3 && q_out.is_contiguous() && k_cache.dim() == 4 && k_cache.is_contiguous() &&
                  v_cache.dim() == 4 && v_cache.is_contiguous() && q.dim() == 2 && k.dim() == 2,
              "qk_head_norm ranks");
  a.T = (int)q_out.size(0);
  a.H = (int)q_out.size(1);
  a.KP = (int)q_out.size(2);
  a.G = (int)k_cache.size(1);
  a.BS = (int)k_cache.size(2);
  a.VP = (int)v_cache.size(3);
  a.D = (int)D;
  a.V = (int)V;
  TORCH_CHECK(k_cache.size(3) == a.KP && v_cache.size(0) == k_cache.size(0) && v_cache.size(1) == a.G && v_cache.size(2) == a.BS,
              "caches must be [NB, G, BS, KP] and [NB, G, BS, VP]");
  TORCH_CHECK(D >= 1 && D <= a.KP && V >= 1 && V <= a.VP && a.KP % 8 == 0, "head sizes");
  TORCH_CHECK(q.size(0) == a.T && q.size(1) == a.H * D && k.size(0) == a.T && k.size(1) == a.G * D, "q [T, H * D], k [T, G * D]");
  a.q = q.data_ptr();
  a.k = k.data_ptr();
  a.ldq = q.stride(0);
  a.ldk = k.stride(0);
  if (v) {
    like(*v, q, "v");
    TORCH_CHECK(v->dim() == 2 && v->size(0) == a.T && v->size(1) == a.G * V, "v [T, G * V]");
    a.v = v->data_ptr();
    a.ldv = v->stride(0);
  } else {
    TORCH_CHECK(V == D, "keys as values have the keys' size");
  }
  aligned16(q_out, "q_out");
  aligned16(k_cache, "k_cache");
  aligned16(v_cache, "v_cache");
  a.q_w = f32_of(q_w, D, "q_w");
  a.k_w = f32_of(k_w, D, "k_w");
  aligned16(q_w, "q_w");
  aligned16(k_w, "k_w");
  a.eps = (float)eps;
  TORCH_CHECK(cos_sin.dim() == 2, "cos_sin must be [max_pos, R]");
  a.cos_sin = f32_of(cos_sin, cos_sin.numel(), "cos_sin");
  aligned16(cos_sin, "cos_sin");
  a.R = (int)cos_sin.size(1);
  TORCH_CHECK(a.R % 2 == 0 && a.R <= D, "rotated dims must be even and at most the head size");
  a.pos = i32_of(pos, "pos");
  a.slots = i32_of(slots, "slots");
  TORCH_CHECK(pos.numel() == a.T && slots.numel() == a.T, "pos / slots length");
  a.q_out = q_out.data_ptr();
  a.k_cache = k_cache.data_ptr();
  a.v_cache = v_cache.data_ptr();
  c10::DeviceGuard g(q.device());
  mlop::launch_qk_head_norm(a, f32, cur());
}

// decode tiles (one query token each) and prompt tiles (128 tokens of a head) of one step.  k, v: paged
// caches [NB, G, 16, KP]; or, with xbase, dense rows [rows, G, KP] of prompt tiles.  by_tile: q [tiles, H,
// KP] and out by decode tile
void attention_hd(Tensor out, Tensor part_o, Tensor part_ml, Tensor part_sem, Tensor q, Tensor k_cache, Tensor v_cache,
                  Tensor block_tables, Tensor tile_seq, Tensor tile_q0, Tensor ptile_seq, Tensor ptile_q0,
                  Tensor q_start, Tensor q_len, Tensor ctx_len, int64_t D, double scale, OptT sink, OptT gate,
                  int64_t part_tokens, int64_t nparts, int64_t window, OptT xbase, bool by_tile, OptT rot, int64_t rot_lo) {
  mlop::AttnHdArgs a{};
  const bool f32 = model_f32(q, "q");
  like(out, q, "out");
  like(k_cache, q, "k_cache");
  like(v_cache, q, "v_cache");
  const int64_t num_tiles = tile_seq.numel(), num_ptiles = ptile_seq.numel();
  TORCH_CHECK(q.dim() == 3 && out.dim() == 3 && out.stride(1) == out.size(2), "q, out ranks");
  a.out_row = out.stride(0);
  TORCH_CHECK(a.out_row >= out.size(1) * out.size(2) && (a.out_row % 8 == 0 || out.is_contiguous()), "out rows");
  a.H = (int)q.size(1);
  a.KP = (int)q.size(2);
  a.V = (int)out.size(2);
  a.D = (int)D;
  a.q_row = q.stride(0);
  a.q_head = q.stride(1);
  const int kd = (int)k_cache.dim();
  TORCH_CHECK(kd == (xbase ? 3 : 4) && v_cache.dim() == kd, "key / value ranks");
  a.G = (int)k_cache.size(1);
  a.VP = (int)v_cache.size(kd - 1);
  TORCH_CHECK(out.size(1) == a.H && out.size(0) == q.size(0), "out must be [T, H, V]");
  TORCH_CHECK(a.KP % 64 == 0 && a.VP % 64 == 0 && D >= 1 && D <= a.KP && a.V >= 1 && a.V <= a.VP &&
                  a.VP <= mlop::kHdMaxV && D <= 4096,
              "head sizes");
  TORCH_CHECK(k_cache.size(kd - 1) == a.KP && v_cache.size(0) == k_cache.size(0) && v_cache.size(1) == a.G, "key / value sizes");
  TORCH_CHECK(a.G >= 1 && a.H % a.G == 0, "query heads must be a multiple of kv heads");
  if (xbase) {
    TORCH_CHECK(num_tiles == 0 && !by_tile, "dense keys are for prompt tiles");
    a.xbase = i32_of(*xbase, "xbase");
    TORCH_CHECK(xbase->numel() >= q_len.numel(), "xbase length");
    a.k_pitch = a.k_row = k_cache.stride(0);
    a.v_pitch = a.v_row = v_cache.stride(0);
    a.k_head = k_cache.stride(1);
    a.v_head = v_cache.stride(1);
    TORCH_CHECK(a.k_row % 8 == 0 && a.v_row % 8 == 0 && a.k_head % 8 == 0 && a.v_head % 8 == 0, "16-B aligned rows");
  } else {
    TORCH_CHECK(k_cache.is_contiguous() && v_cache.is_contiguous() && k_cache.size(2) == 16 && v_cache.size(2) == 16,
                "caches must be [NB, G, 16, KP] and [NB, G, 16, VP]");
    a.k_pitch = (long)a.G * a.KP;
    a.v_pitch = (long)a.G * a.VP;
    a.k_row = a.KP;
    a.v_row = a.VP;
    a.k_head = 16l * a.KP;
    a.v_head = 16l * a.VP;
  }
  TORCH_CHECK(!by_tile || (num_ptiles == 0 && q.size(0) >= num_tiles), "by_tile is for decode tiles");
  TORCH_CHECK(a.q_row % 8 == 0 && a.q_head % 8 == 0, "16-B aligned query rows");
  TORCH_CHECK(scale > 0, "score scale must be positive");
  TORCH_CHECK(window >= 0 && window < (1 << 30), "window");
  a.window = (int)window;
  a.by_tile = by_tile;
  for (const Tensor* t : {&q, &k_cache, &v_cache, &out}) aligned16(*t, "attention operand");
  a.bt = i32_of(block_tables, "block_tables");
  a.bt_stride = (int)block_tables.stride(0);
  a.q_start = i32_of(q_start, "q_start");
  a.q_len = i32_of(q_len, "q_len");
  a.ctx_len = i32_of(ctx_len, "ctx_len");
  TORCH_CHECK(q_start.numel() == q_len.numel() && q_len.numel() == ctx_len.numel() && block_tables.size(0) >= q_len.numel(),
              "per-sequence arrays");
  TORCH_CHECK(tile_seq.numel() == tile_q0.numel() && ptile_seq.numel() == ptile_q0.numel(), "tile arrays");
  if (sink) a.sink = f32_of(*sink, a.H, "sink");
  if (gate) {
    like(*gate, q, "gate");
    TORCH_CHECK(gate->dim() == 2 && !by_tile && gate->size(0) == q.size(0) &&
                    (gate->size(1) == a.H || gate->size(1) == (int64_t)a.H * a.V),
                "gate must be [T, H] or [T, H * V]");
    a.gate = gate->data_ptr();
    a.gate_stride = gate->stride(0);
    a.gate_elem = gate->size(1) != a.H;
    a.gate_vec = a.V % 4 == 0 && a.gate_stride % 4 == 0 && reinterpret_cast<uintptr_t>(a.gate) % 8 == 0;
  }
  if (rot) {
    a.n_rot = (int)rot->size(1);
    a.n_pos = (int)rot->size(0);
    a.rot = f32_of(*rot, rot->numel(), "rot");
    a.rot_lo = (int)rot_lo;
    TORCH_CHECK(num_tiles == 0 && rot->dim() == 2 && a.n_pos >= 1 && a.n_rot % 2 == 0 && rot_lo >= 0 && rot_lo % 8 == 0 &&
                    rot_lo + a.n_rot <= a.D,
                "rot [positions, rotated dims] of prompt tiles");
  }
  a.scale_log2 = (float)(scale * 1.4426950408889634);
  a.num_blocks = (int)k_cache.size(0);
  a.out = out.data_ptr();
  a.q = q.data_ptr();
  a.k_cache = k_cache.data_ptr();
  a.v_cache = v_cache.data_ptr();
  const bool latent = mlop::latent_decode_ok(a, f32);
  const bool plain = f32 || ((a.KP > mlop::kHdMaxDim || a.VP > mlop::kHdMaxDim) && !latent);
  TORCH_CHECK(part_tokens > 0 && part_tokens % 32 == 0 && nparts >= 1, "partition size");
  float *po = nullptr, *pml = nullptr;
  int* sem = nullptr;
  if (nparts > 1 && num_tiles && !plain) {
    // 16-head groups (the latent kernel: pairs of them)
    const int64_t units = num_tiles * (latent ? (a.H + 31) / 32 * 2 : a.G * ((a.H / a.G + 15) / 16));
    TORCH_CHECK(part_o.scalar_type() == at::kFloat && part_ml.scalar_type() == at::kFloat &&
                    part_o.numel() >= units * nparts * 16 * a.VP && part_ml.numel() >= units * nparts * 16 * 2,
                "partial workspace too small");
    i32_of(part_sem, "part_sem");
    TORCH_CHECK(part_sem.numel() >= units, "part_sem too small");
    po = part_o.data_ptr<float>();
    pml = part_ml.data_ptr<float>();
    sem = part_sem.data_ptr<int>();
  }
  c10::DeviceGuard g(q.device());
  mlop::launch_paged_hd(a, f32, po, pml, sem, i32_of(tile_seq, "tile_seq"), i32_of(tile_q0, "tile_q0"), (int)num_tiles,
                        (int)part_tokens, (int)nparts, cur());
  mlop::launch_flash_hd(a, f32, i32_of(ptile_seq, "ptile_seq"), i32_of(ptile_q0, "ptile_q0"), (int)num_ptiles, cur());
}

void gla(Tensor out, Tensor state, Tensor proj, int64_t H, int64_t dk, int64_t dv, Tensor a2, Tensor a2_b, Tensor norm_w,
         double tau, double eps, Tensor q_start, Tensor q_len, Tensor ctx_len, Tensor rows, Tensor item_seq,
         Tensor item_t0, Tensor crow_seq, Tensor crow_item0, int64_t chunk) {
  mlop::GlaArgs a{};
  const bool f32 = model_f32(proj, "proj");
  like(out, proj, "out");
  like(a2, proj, "a2");
  TORCH_CHECK(H >= 1 && dk >= 1 && dv >= 1 && dk <= 4096 && dv <= 4096 && tau != 0.0, "gla sizes");
  TORCH_CHECK(a2.dim() == 2 && a2.is_contiguous() && a2.size(0) == H * dk, "a2 must be [H * dk, rank]");
  a.rank = (int)a2.size(1);
  TORCH_CHECK(proj.dim() == 2 && proj.size(1) >= 2 * H * dk + 2 * H * dv + a.rank, "proj is too narrow");
  const int64_t T = proj.size(0);
  TORCH_CHECK(out.is_contiguous() && out.numel() == T * H * dv, "out must be [T, H * dv]");
  TORCH_CHECK(state.is_cuda() && state.scalar_type() == at::kFloat && state.is_contiguous() && state.dim() == 4 &&
                  state.size(1) == H && state.size(2) == dk && state.size(3) == dv,
              "state must be [slots, H, dk, dv] fp32");
  aligned16(state, "state");
  a.out = out.data_ptr();
  a.proj = proj.data_ptr();
  a.ldp = proj.stride(0);
  a.a2 = a2.data_ptr();
  a.a2_b = f32_of(a2_b, H * dk, "a2_b");
  a.norm_w = f32_of(norm_w, dv, "norm_w");
  a.state = state.data_ptr<float>();
  a.n_slots = (int)state.size(0);
  a.q_start = i32_of(q_start, "q_start");
  a.q_len = i32_of(q_len, "q_len");
  a.ctx_len = i32_of(ctx_len, "ctx_len");
  a.H = (int)H;
  a.dk = (int)dk;
  a.dv = (int)dv;
  a.inv_tau = (float)(1.0 / tau);
  a.q_scale = (float)(1.0 / std::sqrt((double)dk));
  a.eps = (float)eps;
  const size_t lds = (size_t)(a.rank + 3 * dk + dv + 4096) * 4;
  TORCH_CHECK(lds <= 60 * 1024, "gla: sizes past the kernels' LDS");
  c10::DeviceGuard g(proj.device());
  mlop::launch_gla_rows(a, f32, i32_of(rows, "rows"), (int)rows.numel(), cur());
  const int n_items = (int)item_seq.numel(), n_crows = (int)crow_seq.numel();
  if (n_crows == 0) return;
  TORCH_CHECK(item_t0.numel() == n_items && crow_item0.numel() == n_crows && chunk >= 16 && chunk % 16 == 0, "chunk lists");
  if (dk > mlop::kGlaMaxDk) {  // past the chunked kernel's key size: token by token
    mlop::launch_gla_rows(a, f32, i32_of(crow_seq, "crow_seq"), n_crows, cur());
    return;
  }
  const auto f = proj.options().dtype(at::kFloat);
  Tensor cstate = at::empty({n_items, H, dk, dv}, f), cdecay = at::empty({n_items, H, dk}, f), o32;
  if (mlop::gla_chunks_need_o32((int)dv)) o32 = at::empty({T, H * dv}, f);
  mlop::launch_gla_chunks(a, f32, o32.defined() ? o32.data_ptr<float>() : nullptr, cstate.data_ptr<float>(),
                          cdecay.data_ptr<float>(), i32_of(item_seq, "item_seq"), i32_of(item_t0, "item_t0"), n_items,
                          i32_of(crow_seq, "crow_seq"), i32_of(crow_item0, "crow_item0"), n_crows, (int)chunk, cur());
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(mlop, m) {
  m.def("hyper_begin(Tensor(a!) xn, Tensor(b!) streams, Tensor ids, Tensor table, float scale, Tensor w_in, "
        "Tensor norm_w, float eps) -> ()");
  m.def("hyper_step(Tensor(a!) xn, Tensor(b!) streams, Tensor y, Tensor mix, Tensor w_out, Tensor w_in, "
        "Tensor norm_w, float eps, bool store) -> ()");
  m.def("act_columns(Tensor(a!) x, int n0, int epi, float a, float b) -> ()");
  m.def("softcap(Tensor(a!) out, Tensor x, float cap) -> ()");
  m.def("qk_norm_rope(Tensor(a!) q_out, Tensor(b!) k_cache, Tensor(c!) v_cache, Tensor proj, int D, int V, "
        "Tensor? q_w, Tensor? k_w, float eps, Tensor cos_sin, Tensor pos, Tensor slots, Tensor? v_first, Tensor? lam) "
        "-> ()");
  m.def("qk_head_norm(Tensor(a!) q_out, Tensor(b!) k_cache, Tensor(c!) v_cache, Tensor q, Tensor k, Tensor? v, int D, int V, "
        "Tensor q_w, Tensor k_w, float eps, Tensor cos_sin, Tensor pos, Tensor slots) -> ()");
  m.def("attention_hd(Tensor(a!) out, Tensor(b!) part_o, Tensor(c!) part_ml, Tensor(d!) part_sem, Tensor q, "
        "Tensor k_cache, Tensor v_cache, Tensor block_tables, Tensor tile_seq, Tensor tile_q0, Tensor ptile_seq, "
        "Tensor ptile_q0, Tensor q_start, Tensor q_len, Tensor ctx_len, int D, float scale, Tensor? sink, Tensor? gate, "
        "int part_tokens, int nparts, int window=0, Tensor? xbase=None, bool by_tile=False, "
        "Tensor? rot=None, int rot_lo=0) -> ()");
  m.def("gla(Tensor(a!) out, Tensor(b!) state, Tensor proj, int H, int dk, int dv, Tensor a2, Tensor a2_b, "
        "Tensor norm_w, float tau, float eps, Tensor q_start, Tensor q_len, Tensor ctx_len, Tensor rows, "
        "Tensor item_seq, Tensor item_t0, Tensor crow_seq, Tensor crow_item0, int chunk) -> ()");
}

TORCH_LIBRARY_IMPL(mlop, CUDA, m) {
  m.impl("hyper_begin", &hyper_begin);
  m.impl("hyper_step", &hyper_step);
  m.impl("act_columns", &act_columns);
  m.impl("softcap", &softcap);
  m.impl("qk_norm_rope", &qk_norm_rope);
  m.impl("qk_head_norm", &qk_head_norm);
  m.impl("attention_hd", &attention_hd);
  m.impl("gla", &gla);
}
