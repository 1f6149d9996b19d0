// torch.ops.mlop.* registrations of the mixers and norms in mixers.h.  Every op checks types and shapes
// on the host before it launches.
#include <cmath>

#include "bind_util.h"
#include "launch.h"
#include "mixers.h"

namespace {

// a step's row lists; T: tokens the per-token operands hold
mlop::StepRows step_rows(const Tensor& q_start, const Tensor& q_len, const Tensor& ctx_len, const Tensor& rows,
                         const Tensor& item_seq, const Tensor& item_t0, const Tensor& crow_seq, const Tensor& crow_item0,
                         int64_t chunk, int64_t n_slots) {
  mlop::StepRows s{};
  s.q_start = i32_of(q_start, "q_start");
  s.q_len = i32_of(q_len, "q_len");
  s.ctx_len = i32_of(ctx_len, "ctx_len");
  TORCH_CHECK(q_start.numel() == q_len.numel() && q_len.numel() == ctx_len.numel(), "per-sequence arrays");
  s.rows = i32_of(rows, "rows");
  s.n_rows = (int)rows.numel();
  s.item_seq = i32_of(item_seq, "item_seq");
  s.item_t0 = i32_of(item_t0, "item_t0");
  s.n_items = (int)item_seq.numel();
  s.crow_seq = i32_of(crow_seq, "crow_seq");
  s.crow_item0 = i32_of(crow_item0, "crow_item0");
  s.n_crows = (int)crow_seq.numel();
  TORCH_CHECK(item_t0.numel() == s.n_items && crow_item0.numel() == s.n_crows, "chunk lists");
  TORCH_CHECK((s.n_items == 0) == (s.n_crows == 0) && (s.n_items == 0 || (chunk >= 16 && chunk % 16 == 0)), "chunk size");
  s.chunk = (int)chunk;
  s.n_slots = (int)n_slots;
  return s;
}

// [n] or one number
const float* vec_or_one(const Tensor& t, int64_t n, bool& one, const char* name) {
  one = t.numel() == 1 && n != 1;
  aligned16(t, name);
  return f32_of(t, one ? 1 : n, name);
}

void residual_common(mlop::ResidualArgs& a, const Tensor& xn, const Tensor& x, const OptT& norm_w, double eps, int64_t width,
                     const OptT& tanh_a, const OptT& tanh_b) {
  TORCH_CHECK(x.dim() == 2 && x.is_contiguous() && x.is_cuda() && x.scalar_type() == at::kFloat, "x must be [T, W] fp32");
  a.T = (int)x.size(0);
  a.W = (int)x.size(1);
  TORCH_CHECK(a.W >= 1 && a.W <= mlop::kResidualMaxW, "row width 1 .. ", mlop::kResidualMaxW);
  TORCH_CHECK(xn.is_contiguous() && xn.numel() == x.numel(), "xn must be [T, W]");
  a.x = x.data_ptr<float>();
  a.xn = xn.data_ptr();
  if (norm_w) a.norm_w = vec_or_one(*norm_w, a.W, a.norm_one, "norm_w");
  a.eps = (float)eps;
  TORCH_CHECK(tanh_a.has_value() == tanh_b.has_value() && (!tanh_a || norm_w), "a dynamic tanh has alpha, weight and b");
  if (tanh_a) {
    a.tanh_a = f32_of(*tanh_a, 1, "tanh alpha");
    a.tanh_b = f32_of(*tanh_b, a.W, "tanh b");
    aligned16(*tanh_b, "tanh b");
  }
  TORCH_CHECK(width >= 0 && width <= a.W, "width");
  a.n = width ? (int)width : a.W;
  for (const Tensor* t : {&x, &xn}) aligned16(*t, "residual operand");
}

void residual_begin(Tensor xn, Tensor x, Tensor ids, Tensor table, double scale, OptT pos_table, Tensor pos, OptT norm_w,
                    double eps, int64_t width, OptT tanh_a, OptT tanh_b) {
  mlop::ResidualArgs a{};
  const bool f32 = model_f32(table, "table");
  like(xn, table, "xn");
  residual_common(a, xn, x, norm_w, eps, width, tanh_a, tanh_b);
  TORCH_CHECK(ids.is_cuda() && ids.scalar_type() == at::kLong && ids.is_contiguous() && ids.numel() == a.T, "ids int64 [T]");
  TORCH_CHECK(table.dim() == 2 && table.is_contiguous() && table.size(1) == a.W, "table must be [vocab, W]");
  aligned16(table, "table");
  a.ids = ids.data_ptr<int64_t>();
  a.table = table.data_ptr();
  a.vocab = table.size(0);
  a.embed_scale = (float)scale;
  if (pos_table) {
    like(*pos_table, table, "pos_table");
    TORCH_CHECK(pos_table->dim() == 2 && pos_table->is_contiguous() && pos_table->size(1) == a.W, "pos_table [n, W]");
    aligned16(*pos_table, "pos_table");
    a.pos_table = pos_table->data_ptr();
    a.n_pos = pos_table->size(0);
    a.pos = i32_of(pos, "pos");
    TORCH_CHECK(pos.numel() == a.T, "pos length");
  }
  a.store = true;
  c10::DeviceGuard g(table.device());
  mlop::launch_residual(a, f32, cur());
}

void residual_step(Tensor xn, Tensor x, OptT y, OptT post_w, OptT norm_w, double eps, bool store, int64_t width, OptT rows,
                   OptT inv, OptT gate, OptT row_w, OptT self, OptT self_w, OptT tanh_a, OptT tanh_b) {
  mlop::ResidualArgs a{};
  TORCH_CHECK(y || rows, "residual_step needs a sublayer output");
  const bool f32 = model_f32(xn, "xn");
  residual_common(a, xn, x, norm_w, eps, width, tanh_a, tanh_b);
  if (y) {
    like(*y, xn, "y");
    TORCH_CHECK(y->is_contiguous() && y->numel() == x.numel(), "y must be [T, W]");
    aligned16(*y, "y");
    a.y = y->data_ptr();
  }
  if (rows) {
    like(*rows, xn, "rows");
    TORCH_CHECK(rows->dim() == 2 && rows->is_contiguous() && rows->size(1) == a.W, "rows must be [R, W]");
    aligned16(*rows, "rows");
    a.rows = rows->data_ptr();
    TORCH_CHECK(inv && inv->dim() == 2 && inv->size(0) == a.T && inv->numel() <= rows->size(0), "inv must be [T, k]");
    a.inv = i32_of(*inv, "inv");
    a.top = (int)inv->size(1);
    if (gate) a.gate = f32_of(*gate, a.T, "gate");
    if (row_w) a.row_w = f32_of(*row_w, inv->numel(), "row_w");
    if (self) {
      like(*self, xn, "self");
      TORCH_CHECK(self->is_contiguous() && self->numel() == x.numel() && self_w, "self must be [T, W], with weights");
      aligned16(*self, "self");
      a.self = self->data_ptr();
      a.self_w = f32_of(*self_w, a.T, "self_w");
    }
  }
  if (post_w) a.post_w = vec_or_one(*post_w, a.W, a.post_one, "post_w");
  a.store = store;
  c10::DeviceGuard g(xn.device());
  mlop::launch_residual(a, f32, cur());
}

void gated_norm(Tensor out, Tensor y, Tensor gate, Tensor w, int64_t groups, double eps, int64_t act, bool gate_first) {
  mlop::GatedNormArgs a{};
  const bool f32 = model_f32(y, "y");
  like(out, y, "out");
  like(gate, y, "gate");
  TORCH_CHECK(y.dim() == 2 && y.is_contiguous() && out.is_contiguous() && out.numel() == y.numel(), "y, out must be [T, n]");
  a.T = (int)y.size(0);
  a.n = (int)y.size(1);
  TORCH_CHECK(gate.dim() == 2 && gate.size(0) == a.T && gate.size(1) == a.n, "gate must be [T, n]");
  TORCH_CHECK(groups >= 1 && a.n % groups == 0, "groups must divide the row");
  TORCH_CHECK(act == mlop::kGateSilu || act == mlop::kGateSigmoid, "gate activation");
  a.groups = (int)groups;
  a.out = out.data_ptr();
  a.y = y.data_ptr();
  a.gate = gate.data_ptr();
  a.ldg = gate.stride(0);
  a.w = f32_of(w, a.n, "w");
  a.eps = (float)eps;
  a.act = (int)act;
  a.gate_first = gate_first;
  c10::DeviceGuard g(y.device());
  mlop::launch_gated_norm(a, f32, cur());
}

void clamp_glu(Tensor out, Tensor x, double alpha, double limit) {
  const bool f32 = model_f32(x, "x");
  like(out, x, "out");
  TORCH_CHECK(x.dim() == 2 && x.is_contiguous() && out.is_contiguous() && x.size(1) % 32 == 0 &&
                  out.numel() * 2 == x.numel(),
              "x must be [T, 2 I] with columns interleaved in groups of 16, out [T, I]");
  aligned16(x, "x");
  aligned16(out, "out");
  c10::DeviceGuard g(x.device());
  mlop::launch_clamp_glu(out.data_ptr(), x.data_ptr(), (int)x.size(0), (int)(x.size(1) / 2), (float)alpha, (float)limit, f32,
                         cur());
}

void short_conv(Tensor out, Tensor tail, Tensor x, Tensor w, OptT b, Tensor q_start, Tensor q_len, Tensor ctx_len,
                Tensor rows, Tensor item_seq, Tensor item_t0, Tensor crow_seq, Tensor crow_item0, int64_t chunk) {
  mlop::ConvArgs a{};
  const bool f32 = model_f32(x, "x");
  like(out, x, "out");
  TORCH_CHECK(w.dim() == 2, "w must be [C, taps]");
  a.C = (int)w.size(0);
  a.taps = (int)w.size(1);
  TORCH_CHECK(a.taps >= 1 && a.taps <= mlop::kConvMaxTaps, "1 .. ", mlop::kConvMaxTaps, " taps");
  TORCH_CHECK(x.dim() == 2 && x.size(1) == a.C && out.is_contiguous() && out.numel() == x.size(0) * a.C, "x, out must be [T, C]");
  TORCH_CHECK(tail.is_cuda() && tail.scalar_type() == at::kFloat && tail.is_contiguous() && tail.dim() == 3 &&
                  tail.size(1) == a.taps - 1 && tail.size(2) == a.C,
              "tail must be [slots, taps - 1, C] fp32");
  a.out = out.data_ptr();
  a.x = x.data_ptr();
  a.ldx = x.stride(0);
  a.w = f32_of(w, (int64_t)a.C * a.taps, "w");
  if (b) a.b = f32_of(*b, a.C, "b");
  a.tail = tail.data_ptr<float>();
  const auto s = step_rows(q_start, q_len, ctx_len, rows, item_seq, item_t0, crow_seq, crow_item0, chunk, tail.size(0));
  c10::DeviceGuard g(x.device());
  mlop::launch_short_conv(a, s, f32, cur());
}

void ssd(Tensor y, Tensor state, Tensor xbc, Tensor dt, int64_t G, Tensor dt_bias, Tensor a_neg, Tensor d_skip,
         Tensor q_start, Tensor q_len, Tensor ctx_len, Tensor rows, Tensor item_seq, Tensor item_t0, Tensor crow_seq,
         Tensor crow_item0, int64_t chunk) {
  mlop::SsdArgs a{};
  const bool f32 = model_f32(xbc, "xbc");
  like(y, xbc, "y");
  like(dt, xbc, "dt");
  TORCH_CHECK(state.is_cuda() && state.scalar_type() == at::kFloat && state.is_contiguous() && state.dim() == 4,
              "state must be [slots, H, N, V] fp32");
  aligned16(state, "state");
  a.H = (int)state.size(1);
  a.N = (int)state.size(2);
  a.V = (int)state.size(3);
  a.G = (int)G;
  TORCH_CHECK(a.H >= 1 && G >= 1 && a.H % G == 0 && a.N >= 1 && a.N <= 4096 && a.V >= 1 && a.V <= 4096, "ssd sizes");
  TORCH_CHECK(xbc.dim() == 2 && xbc.size(1) == (int64_t)a.H * a.V + 2 * G * a.N, "xbc must be [T, H V + 2 G N]");
  const int64_t T = xbc.size(0);
  TORCH_CHECK(y.is_contiguous() && y.numel() == T * a.H * a.V, "y must be [T, H * V]");
  TORCH_CHECK(dt.dim() == 2 && dt.size(0) == T && dt.size(1) == a.H, "dt must be [T, H]");
  aligned16(xbc, "xbc");
  a.y = y.data_ptr();
  a.xbc = xbc.data_ptr();
  a.ldx = xbc.stride(0);
  a.dt = dt.data_ptr();
  a.ldt = dt.stride(0);
  a.dt_bias = f32_of(dt_bias, a.H, "dt_bias");
  a.a_neg = f32_of(a_neg, a.H, "a_neg");
  a.d_skip = f32_of(d_skip, a.H, "d_skip");
  a.state = state.data_ptr<float>();
  const auto s = step_rows(q_start, q_len, ctx_len, rows, item_seq, item_t0, crow_seq, crow_item0, chunk, state.size(0));
  c10::DeviceGuard g(xbc.device());
  Tensor ws;
  if (s.n_items && a.N <= mlop::kSsdMaxN)
    ws = at::empty({mlop::ssd_ws_floats(s.n_items, s.chunk, a.H)}, xbc.options().dtype(at::kFloat));
  mlop::launch_ssd(a, s, ws.defined() ? ws.data_ptr<float>() : nullptr, f32, cur());
}

void delta(Tensor o, Tensor state, Tensor proj, Tensor w2, Tensor w0, Tensor a_b, double decay_scale, double unit_eps,
           Tensor q_start, Tensor q_len, Tensor ctx_len, Tensor rows, Tensor item_seq, Tensor item_t0, Tensor crow_seq,
           Tensor crow_item0, int64_t chunk) {
  mlop::DeltaArgs a{};
  const bool f32 = model_f32(proj, "proj");
  like(o, proj, "o");
  like(w2, proj, "w2");
  TORCH_CHECK(state.is_cuda() && state.scalar_type() == at::kFloat && state.is_contiguous() && state.dim() == 4,
              "state must be [slots, H, dk, dv] fp32");
  aligned16(state, "state");
  a.H = (int)state.size(1);
  a.dk = (int)state.size(2);
  a.dv = (int)state.size(3);
  TORCH_CHECK(a.H >= 1 && a.dk >= 1 && a.dk <= 1024 && a.dv >= 1 && a.dv <= 4096 && decay_scale >= 0, "delta sizes");
  TORCH_CHECK(w2.dim() == 2 && w2.is_contiguous() && w2.size(0) == (int64_t)a.H * a.dk, "w2 must be [H * dk, rank]");
  a.rank = (int)w2.size(1);
  const int64_t T = proj.size(0);
  TORCH_CHECK(proj.dim() == 2 && proj.size(1) >= (int64_t)a.H * (3 * a.dk + a.dv) + a.rank, "proj is too narrow");
  TORCH_CHECK(o.is_contiguous() && o.numel() == T * a.H * a.dv, "o must be [T, H * dv]");
  TORCH_CHECK((size_t)(a.rank + 5 * a.dk + 3 * 512 * 4) * 4 <= 60 * 1024, "delta: sizes past the kernels' LDS");
  aligned16(proj, "proj");
  aligned16(w2, "w2");
  a.o = o.data_ptr();
  a.proj = proj.data_ptr();
  a.ldp = proj.stride(0);
  a.w2 = w2.data_ptr();
  a.w0 = f32_of(w0, (int64_t)a.H * a.dk, "w0");
  a.a_b = f32_of(a_b, (int64_t)a.H * a.dk, "a_b");
  a.state = state.data_ptr<float>();
  a.decay_scale = (float)decay_scale;
  a.unit_eps = (float)unit_eps;
  const auto s = step_rows(q_start, q_len, ctx_len, rows, item_seq, item_t0, crow_seq, crow_item0, chunk, state.size(0));
  c10::DeviceGuard g(proj.device());
  Tensor ws;
  if (s.n_items && mlop::delta_blocks_ok(a.dk, a.decay_scale))
    ws = at::empty({mlop::delta_ws_floats(s.n_items, s.chunk, a.H, a.dk)}, proj.options().dtype(at::kFloat));
  mlop::launch_delta(a, s, ws.defined() ? ws.data_ptr<float>() : nullptr, f32, cur());
}

// the query latents' part of the arguments
void query_part(mlop::LatentStoreArgs& a, const Tensor& out, const Tensor& x, const Tensor& w) {
  like(out, x, "q_out");
  TORCH_CHECK(x.dim() == 2 && out.dim() == 2 && out.is_contiguous() && out.size(0) == x.size(0) && out.size(1) >= x.size(1),
              "query latents must be [T, r], out [T, >= r]");
  aligned16(out, "q_out");
  a.q_out = out.data_ptr();
  a.q = x.data_ptr();
  a.ldq = x.stride(0);
  a.QR = (int)x.size(1);
  a.QP = (int)out.size(1);
  a.q_w = f32_of(w, a.QR, "q_w");
  a.T = (int)x.size(0);
}

void latent_store(Tensor cache, Tensor l, Tensor w, double eps, Tensor slots, OptT k, OptT table, OptT pos, int64_t off,
                  OptT q_out, OptT q, OptT q_w) {
  mlop::LatentStoreArgs a{};
  const bool f32 = model_f32(l, "l");
  like(cache, l, "cache");
  TORCH_CHECK(cache.dim() == 4 && cache.is_contiguous() && cache.size(1) == 1, "cache must be [NB, 1, BS, RP]");
  TORCH_CHECK(l.dim() == 2 && l.size(1) <= cache.size(3) && slots.numel() == l.size(0), "latents must be [T, R]");
  aligned16(cache, "cache");
  if (q) {
    TORCH_CHECK(q_out && q_w && q->size(0) == l.size(0), "query latents");
    like(*q, l, "q");
    query_part(a, *q_out, *q, *q_w);
  }
  a.cache = cache.data_ptr();
  a.l = l.data_ptr();
  a.ldl = l.stride(0);
  a.R = (int)l.size(1);
  a.RP = (int)cache.size(3);
  a.w = f32_of(w, a.R, "w");
  a.slots = i32_of(slots, "slots");
  a.eps = (float)eps;
  a.T = (int)l.size(0);
  if (k) {
    like(*k, l, "k");
    TORCH_CHECK(table && pos && table->dim() == 2 && k->dim() == 2 && k->size(0) == a.T, "rotated keys");
    a.n_rot = (int)table->size(1);
    a.n_pos = (int)table->size(0);
    TORCH_CHECK(k->size(1) == a.n_rot && a.n_rot % 2 == 0 && a.n_pos >= 1 && off >= a.R && off + a.n_rot <= a.RP, "rotated key size");
    a.k = k->data_ptr();
    a.ldk = k->stride(0);
    a.table = f32_of(*table, table->numel(), "table");
    a.pos = i32_of(*pos, "pos");
    TORCH_CHECK(pos->numel() == a.T, "pos length");
    a.off = (int)off;
  }
  c10::DeviceGuard g(l.device());
  mlop::launch_latent_store(a, f32, cur());
}

void latent_query(Tensor out, Tensor x, Tensor w, double eps) {
  mlop::LatentStoreArgs a{};
  const bool f32 = model_f32(x, "x");
  query_part(a, out, x, w);
  a.eps = (float)eps;
  c10::DeviceGuard g(x.device());
  mlop::launch_latent_store(a, f32, cur());
}

void latent_gather(Tensor out, Tensor cache, Tensor block_tables, Tensor xbase, Tensor q_len, Tensor ctx_len,
                   Tensor crow_seq, int64_t rows, int64_t x_max, int64_t window) {
  mlop::LatentGatherArgs a{};
  const bool f32 = model_f32(cache, "cache");
  like(out, cache, "out");
  TORCH_CHECK(cache.dim() == 4 && cache.is_contiguous() && cache.size(1) == 1, "cache must be [NB, 1, BS, RP]");
  a.RP = (int)cache.size(3);
  TORCH_CHECK(out.dim() == 2 && out.is_contiguous() && out.size(1) == a.RP && out.size(0) >= rows && a.RP % 64 == 0,
              "out must be [rows + pad, RP]");
  aligned16(out, "out");
  aligned16(cache, "cache");
  a.out = out.data_ptr();
  a.cache = cache.data_ptr();
  a.bt = i32_of(block_tables, "block_tables");
  a.bt_stride = (int)block_tables.stride(0);
  a.xbase = i32_of(xbase, "xbase");
  a.q_len = i32_of(q_len, "q_len");
  a.ctx_len = i32_of(ctx_len, "ctx_len");
  a.crow_seq = i32_of(crow_seq, "crow_seq");
  a.n_crows = (int)crow_seq.numel();
  a.x_max = (int)x_max;
  a.rows = (int)rows;
  a.pad = (int)(out.size(0) - rows);
  a.BS = (int)cache.size(2);
  a.num_blocks = (int)cache.size(0);
  a.window = (int)window;
  c10::DeviceGuard g(cache.device());
  mlop::launch_latent_gather(a, f32, cur());
}

void head_mm(Tensor out, Tensor x, Tensor w, Tensor tile_seq, Tensor tile_q0, Tensor q_start, Tensor q_len, bool x_tok,
             bool out_tok, OptT gate, OptT table, OptT pos, int64_t x_off) {
  mlop::HeadMmArgs a{};
  const bool f32 = model_f32(x, "x");
  like(out, x, "out");
  like(w, x, "w");
  TORCH_CHECK(w.dim() == 3 && w.is_contiguous() && x.dim() == 3 && out.dim() == 3, "w [H, N, K], x [rows, H, K], out [rows, H, N]");
  a.H = (int)w.size(0);
  a.N = (int)w.size(1);
  a.K = (int)w.size(2);
  TORCH_CHECK(a.K % 64 == 0 && x.size(1) == a.H && x.size(2) >= a.K && out.size(1) == a.H &&
                  (table ? out.size(2) > a.N && (out.size(2) - a.N) % 2 == 0 : out.size(2) == a.N),
              "head_mm sizes");
  a.n_tiles = (int)tile_seq.numel();
  TORCH_CHECK((x_tok || x.size(0) >= a.n_tiles) && (out_tok || out.size(0) >= a.n_tiles) && a.n_tiles <= 65535, "head_mm rows");
  a.out = out.data_ptr();
  a.x = x.data_ptr();
  a.w = w.data_ptr();
  a.ldx = x.stride(0);
  a.hx = x.stride(1);
  a.ldo = out.stride(0);
  a.ho = out.stride(1);
  TORCH_CHECK(a.ldx % 8 == 0 && a.hx % 8 == 0, "16-B aligned rows");
  aligned16(x, "x");
  aligned16(w, "w");
  a.tile_seq = i32_of(tile_seq, "tile_seq");
  a.tile_q0 = i32_of(tile_q0, "tile_q0");
  a.q_start = i32_of(q_start, "q_start");
  a.q_len = i32_of(q_len, "q_len");
  a.x_tok = x_tok;
  a.out_tok = out_tok;
  if (table) {
    a.n_rot = (int)table->size(1);
    a.n_pos = (int)table->size(0);
    a.extra = (int)out.size(2) - a.N;
    TORCH_CHECK(pos && table->dim() == 2 && a.n_pos >= 1 && a.n_rot % 2 == 0 && a.n_rot <= a.extra && x_off >= 0 &&
                    x_off + a.n_rot <= x.size(2),
                "rotated query part");
    a.table = f32_of(*table, table->numel(), "table");
    a.pos = i32_of(*pos, "pos");
    a.x_off = (int)x_off;
  }
  if (gate) {
    like(*gate, x, "gate");
    TORCH_CHECK(gate->dim() == 2 && gate->size(1) == (int64_t)a.H * a.N, "gate must be [T, H * N]");
    a.gate = gate->data_ptr();
    a.ldg = gate->stride(0);
  }
  c10::DeviceGuard g(x.device());
  mlop::launch_head_mm(a, f32, cur());
}

// operands common to the forms of the routing kinds
struct SigShape {
  int T, E, rows, k, H;
  float *topw, *gate;
  int *topi, *inv;
};
SigShape sig_shape(const Tensor& topw, const Tensor& topi, const Tensor& inv, const OptT& gate, int64_t T, int64_t H, int64_t rows,
                   int64_t E) {
  SigShape s{};
  const int64_t k = topi.dim() == 2 ? topi.size(1) : 0;
  TORCH_CHECK(E >= 1 && E <= mlop::kSigMaxE && k >= 1 && k <= E && k <= mlop::kSigMaxTop, "1 .. ", mlop::kSigMaxE, " experts, top 1 .. ",
              mlop::kSigMaxTop);
  TORCH_CHECK(rows == E + (gate ? 1 : 0), "router rows: the experts', then the gate's");
  TORCH_CHECK(topi.size(0) == T && inv.numel() == T * k && T * k < (1 << 28), "topi, inv must be [T, k]");
  s.T = (int)T, s.E = (int)E, s.rows = (int)rows, s.k = (int)k, s.H = (int)H;
  s.topw = const_cast<float*>(f32_of(topw, T * k, "topw"));
  s.topi = const_cast<int*>(i32_of(topi, "topi"));
  s.inv = const_cast<int*>(i32_of(inv, "inv"));
  if (gate) s.gate = const_cast<float*>(f32_of(*gate, T, "gate"));
  return s;
}
int* offsets_of(const Tensor& offsets, int64_t E) {
  TORCH_CHECK(offsets.numel() == E + 1, "offsets must be [E + 1]");
  return const_cast<int*>(i32_of(offsets, "offsets"));
}
void router_rows(const Tensor& x, const Tensor& w) {
  TORCH_CHECK(x.is_cuda() && x.scalar_type() == at::kBFloat16 && w.is_cuda() && w.scalar_type() == at::kBFloat16, "bf16 x, router");
  TORCH_CHECK(x.dim() == 2 && x.is_contiguous() && w.dim() == 2 && w.is_contiguous() && w.size(1) == x.size(1) && x.size(1) % 8 == 0,
              "x must be [T, H], router [rows, H], H a multiple of 8");
  aligned16(x, "x");
  aligned16(w, "router");
}

void moe_dispatch_small_sigmoid(Tensor topw, Tensor topi, Tensor xp, Tensor offsets, Tensor src, Tensor inv, OptT gate, Tensor x,
                                Tensor w, int64_t E) {
  router_rows(x, w);
  const auto s = sig_shape(topw, topi, inv, gate, x.size(0), x.size(1), w.size(0), E);
  TORCH_CHECK(s.T >= 1 && s.T <= 16, "1 .. 16 tokens");
  like(xp, x, "xp");
  TORCH_CHECK(xp.is_contiguous() && xp.dim() == 2 && xp.size(0) == s.T * s.k && xp.size(1) == s.H && src.numel() == s.T * s.k, "xp [T * k, H]");
  aligned16(xp, "xp");
  c10::DeviceGuard g(x.device());
  mlop::launch_moe_dispatch_small_sigmoid(s.topw, s.topi, xp.data_ptr(), offsets_of(offsets, E), const_cast<int*>(i32_of(src, "src")),
                                          s.inv, s.gate, x.data_ptr(), w.data_ptr(), s.T, s.E, s.rows, s.k, s.H, cur());
}

void moe_dispatch_mid_sigmoid(Tensor topw, Tensor topi, Tensor offsets, Tensor a_rows, Tensor row_w, Tensor inv, OptT gate, Tensor x,
                              Tensor w, int64_t E) {
  router_rows(x, w);
  const auto s = sig_shape(topw, topi, inv, gate, x.size(0), x.size(1), w.size(0), E);
  TORCH_CHECK(s.T >= 1 && a_rows.numel() == s.T * s.k, "a_rows must be [T * k]");
  c10::DeviceGuard g(x.device());
  mlop::launch_moe_dispatch_mid_sigmoid(s.topw, s.topi, offsets_of(offsets, E), const_cast<int*>(i32_of(a_rows, "a_rows")),
                                        const_cast<float*>(f32_of(row_w, (int64_t)s.T * s.k, "row_w")), s.inv, s.gate, x.data_ptr(),
                                        w.data_ptr(), s.T, s.E, s.rows, s.k, s.H, cur());
}

void moe_route_sigmoid(Tensor topw, Tensor topi, OptT gate, Tensor logits, int64_t E) {
  TORCH_CHECK(logits.dim() == 2, "logits must be [T, rows]");
  const auto s = sig_shape(topw, topi, topi, gate, logits.size(0), 0, logits.size(1), E);
  c10::DeviceGuard g(logits.device());
  mlop::launch_moe_route_sigmoid(s.topw, s.topi, s.gate, f32_of(logits, logits.numel(), "logits"), s.T, s.E, s.rows, s.k, cur());
}

// the choice among all of the router's outputs, the first E of them experts
mlop::ChooseArgs choose_args(const OptT& correction, const OptT& self_w, int64_t T, int64_t n, int64_t E, int64_t k, int64_t groups,
                             int64_t keep) {
  TORCH_CHECK(n >= E && n <= mlop::kSigMaxE, "router outputs: E .. ", mlop::kSigMaxE);
  TORCH_CHECK(groups >= 1 && n % groups == 0 && keep >= 1 && keep <= groups && k <= n / groups * keep,
              "groups must divide the outputs, the kept ones hold the choice");
  TORCH_CHECK(self_w.has_value() == (n > E), "self_w comes with identity experts");
  mlop::ChooseArgs c{};
  c.n = (int)n, c.groups = (int)groups, c.keep = (int)keep;
  if (correction) c.correction = f32_of(*correction, n, "correction");
  if (self_w) c.self_w = const_cast<float*>(f32_of(*self_w, T, "self_w"));
  return c;
}
// as sig_shape; top may exceed the experts where identity experts are chosen beside them
SigShape group_shape(const Tensor& topw, const Tensor& topi, const Tensor& inv, int64_t T, int64_t H, int64_t rows, int64_t E) {
  TORCH_CHECK(E >= 1 && E <= rows, "1 .. rows experts");
  SigShape s = sig_shape(topw, topi, inv, std::nullopt, T, H, rows, rows);
  s.E = (int)E;
  return s;
}

void moe_dispatch_small_groups(Tensor topw, Tensor topi, Tensor xp, Tensor offsets, Tensor src, Tensor inv, OptT self_w, Tensor x,
                               Tensor w, OptT correction, int64_t E, int64_t groups, int64_t keep) {
  router_rows(x, w);
  const auto s = group_shape(topw, topi, inv, x.size(0), x.size(1), w.size(0), E);
  const auto c = choose_args(correction, self_w, s.T, s.rows, E, s.k, groups, keep);
  TORCH_CHECK(s.T >= 1 && s.T <= 16, "1 .. 16 tokens");
  like(xp, x, "xp");
  TORCH_CHECK(xp.is_contiguous() && xp.dim() == 2 && xp.size(0) == s.T * s.k && xp.size(1) == s.H && src.numel() == s.T * s.k, "xp [T * k, H]");
  aligned16(xp, "xp");
  c10::DeviceGuard g(x.device());
  mlop::launch_moe_dispatch_small_groups(s.topw, s.topi, xp.data_ptr(), offsets_of(offsets, E), const_cast<int*>(i32_of(src, "src")),
                                         s.inv, x.data_ptr(), w.data_ptr(), s.T, s.E, s.k, s.H, c, cur());
}

void moe_dispatch_mid_groups(Tensor topw, Tensor topi, Tensor offsets, Tensor a_rows, Tensor inv, OptT self_w, Tensor x, Tensor w,
                             OptT correction, int64_t E, int64_t groups, int64_t keep) {
  router_rows(x, w);
  const auto s = group_shape(topw, topi, inv, x.size(0), x.size(1), w.size(0), E);
  const auto c = choose_args(correction, self_w, s.T, s.rows, E, s.k, groups, keep);
  TORCH_CHECK(s.T >= 1 && a_rows.numel() == s.T * s.k, "a_rows must be [T * k]");
  c10::DeviceGuard g(x.device());
  mlop::launch_moe_dispatch_mid_groups(s.topw, s.topi, offsets_of(offsets, E), const_cast<int*>(i32_of(a_rows, "a_rows")), s.inv,
                                       x.data_ptr(), w.data_ptr(), s.T, s.E, s.k, s.H, c, cur());
}

void moe_route_groups(Tensor topw, Tensor topi, OptT self_w, Tensor logits, OptT correction, int64_t E, int64_t groups, int64_t keep) {
  TORCH_CHECK(logits.dim() == 2, "logits must be [T, rows]");
  const auto s = group_shape(topw, topi, topi, logits.size(0), 0, logits.size(1), E);
  const auto c = choose_args(correction, self_w, s.T, s.rows, E, s.k, groups, keep);
  c10::DeviceGuard g(logits.device());
  mlop::launch_moe_route_groups(s.topw, s.topi, f32_of(logits, logits.numel(), "logits"), s.T, s.E, s.k, c, cur());
}

// fp32: the experts' rows gathered, times their scores (topw; none: as they are)
void moe_permute_scaled(Tensor xp, Tensor offsets, Tensor src, Tensor inv, Tensor x, Tensor topi, OptT topw, int64_t E) {
  TORCH_CHECK(x.dim() == 2 && topi.dim() == 2 && topi.size(0) == x.size(0) && E >= 1 && E <= mlop::kSigMaxE, "x [T, H], topi [T, k]");
  const int64_t T = x.size(0), k = topi.size(1), H = x.size(1);
  TORCH_CHECK(src.numel() == T * k && inv.numel() == T * k && T * k < (1 << 28), "src, inv must be [T * k]");
  c10::DeviceGuard g(x.device());
  mlop::launch_moe_permute_scaled(const_cast<float*>(f32_of(xp, T * k * H, "xp")), offsets_of(offsets, E),
                                  const_cast<int*>(i32_of(src, "src")), const_cast<int*>(i32_of(inv, "inv")), f32_of(x, x.numel(), "x"),
                                  i32_of(topi, "topi"), topw ? f32_of(*topw, T * k, "topw") : nullptr, (int)T, (int)k, (int)H, (int)E,
                                  cur());
}

void grouped_plain(Tensor out, Tensor a, Tensor w, Tensor offsets) {
  TORCH_CHECK(a.dim() == 2 && w.dim() == 3 && out.dim() == 2 && w.size(2) == a.size(1) && out.size(0) == a.size(0) &&
                  out.size(1) == w.size(1) && a.size(0) < (1 << 20),
              "a [R, K], w [G, N, K], out [R, N]");
  c10::DeviceGuard g(a.device());
  mlop::launch_grouped_plain(const_cast<float*>(f32_of(out, out.numel(), "out")), f32_of(a, a.numel(), "a"), f32_of(w, w.numel(), "w"),
                             offsets_of(offsets, w.size(0)), (int)w.size(0), (int)a.size(0), (int)w.size(1), (int)w.size(2), cur());
}

}  // namespace

#define MLOP_ROWS                                                                                                \
  "Tensor q_start, Tensor q_len, Tensor ctx_len, Tensor rows, Tensor item_seq, Tensor item_t0, Tensor crow_seq, " \
  "Tensor crow_item0, int chunk"

TORCH_LIBRARY_FRAGMENT(mlop, m) {
  m.def("residual_begin(Tensor(a!) xn, Tensor(b!) x, Tensor ids, Tensor table, float scale, Tensor? pos_table, Tensor pos, "
        "Tensor? norm_w, float eps, int width=0, Tensor? tanh_a=None, Tensor? tanh_b=None) -> ()");
  m.def("residual_step(Tensor(a!) xn, Tensor(b!) x, Tensor? y, Tensor? post_w, Tensor? norm_w, float eps, bool store, "
        "int width=0, Tensor? rows=None, Tensor? inv=None, Tensor? gate=None, Tensor? row_w=None, Tensor? self_x=None, "
        "Tensor? self_w=None, Tensor? tanh_a=None, Tensor? tanh_b=None) -> ()");
  m.def("gated_norm(Tensor(a!) out, Tensor y, Tensor gate, Tensor w, int groups, float eps, int act, bool gate_first) -> ()");
  m.def("clamp_glu(Tensor(a!) out, Tensor x, float alpha, float limit) -> ()");
  m.def("short_conv(Tensor(a!) out, Tensor(b!) tail, Tensor x, Tensor w, Tensor? b, " MLOP_ROWS ") -> ()");
  m.def("ssd(Tensor(a!) y, Tensor(b!) state, Tensor xbc, Tensor dt, int G, Tensor dt_bias, Tensor a_neg, Tensor d_skip, "
        MLOP_ROWS ") -> ()");
  m.def("delta(Tensor(a!) o, Tensor(b!) state, Tensor proj, Tensor w2, Tensor w0, Tensor a_b, float decay_scale, "
        "float unit_eps, " MLOP_ROWS ") -> ()");
  m.def("latent_store(Tensor(a!) cache, Tensor l, Tensor w, float eps, Tensor slots, Tensor? k=None, Tensor? table=None, "
        "Tensor? pos=None, int off=0, Tensor(b!)? q_out=None, Tensor? q=None, Tensor? q_w=None) -> ()");
  m.def("latent_query(Tensor(a!) out, Tensor x, Tensor w, float eps) -> ()");
  m.def("latent_gather(Tensor(a!) out, Tensor cache, Tensor block_tables, Tensor xbase, Tensor q_len, Tensor ctx_len, "
        "Tensor crow_seq, int rows, int x_max, int window) -> ()");
  m.def("head_mm(Tensor(a!) out, Tensor x, Tensor w, Tensor tile_seq, Tensor tile_q0, Tensor q_start, Tensor q_len, "
        "bool x_tok, bool out_tok, Tensor? gate, Tensor? table=None, Tensor? pos=None, int x_off=0) -> ()");
  m.def("moe_dispatch_small_sigmoid(Tensor(a!) topw, Tensor(b!) topi, Tensor(c!) xp, Tensor(d!) offsets, Tensor(e!) src, "
        "Tensor(f!) inv, Tensor(g!)? gate, Tensor x, Tensor router, int n_experts) -> ()");
  m.def("moe_dispatch_mid_sigmoid(Tensor(a!) topw, Tensor(b!) topi, Tensor(c!) offsets, Tensor(d!) a_rows, Tensor(e!) row_w, "
        "Tensor(f!) inv, Tensor(g!)? gate, Tensor x, Tensor router, int n_experts) -> ()");
  m.def("moe_route_sigmoid(Tensor(a!) topw, Tensor(b!) topi, Tensor(c!)? gate, Tensor logits, int n_experts) -> ()");
  m.def("moe_dispatch_small_groups(Tensor(a!) topw, Tensor(b!) topi, Tensor(c!) xp, Tensor(d!) offsets, Tensor(e!) src, "
        "Tensor(f!) inv, Tensor(g!)? self_w, Tensor x, Tensor router, Tensor? correction, int n_experts, int groups, int keep) -> ()");
  m.def("moe_dispatch_mid_groups(Tensor(a!) topw, Tensor(b!) topi, Tensor(c!) offsets, Tensor(d!) a_rows, Tensor(e!) inv, "
        "Tensor(f!)? self_w, Tensor x, Tensor router, Tensor? correction, int n_experts, int groups, int keep) -> ()");
  m.def("moe_route_groups(Tensor(a!) topw, Tensor(b!) topi, Tensor(c!)? self_w, Tensor logits, Tensor? correction, int n_experts, "
        "int groups, int keep) -> ()");
  m.def("moe_permute_scaled(Tensor(a!) xp, Tensor(b!) offsets, Tensor(c!) src, Tensor(d!) inv, Tensor x, Tensor topi, Tensor? topw, "
        "int n_experts) -> ()");
  m.def("grouped_plain(Tensor(a!) out, Tensor a, Tensor w, Tensor offsets) -> ()");
}

TORCH_LIBRARY_IMPL(mlop, CUDA, m) {
  m.impl("residual_begin", &residual_begin);
  m.impl("residual_step", &residual_step);
  m.impl("gated_norm", &gated_norm);
  m.impl("clamp_glu", &clamp_glu);
  m.impl("short_conv", &short_conv);
  m.impl("ssd", &ssd);
  m.impl("delta", &delta);
  m.impl("latent_store", &latent_store);
  m.impl("latent_query", &latent_query);
  m.impl("latent_gather", &latent_gather);
  m.impl("head_mm", &head_mm);
  m.impl("moe_dispatch_small_sigmoid", &moe_dispatch_small_sigmoid);
  m.impl("moe_dispatch_mid_sigmoid", &moe_dispatch_mid_sigmoid);
  m.impl("moe_route_sigmoid", &moe_route_sigmoid);
  m.impl("moe_dispatch_small_groups", &moe_dispatch_small_groups);
  m.impl("moe_dispatch_mid_groups", &moe_dispatch_mid_groups);
  m.impl("moe_route_groups", &moe_route_groups);
  m.impl("moe_permute_scaled", &moe_permute_scaled);
  m.impl("grouped_plain", &grouped_plain);
}
