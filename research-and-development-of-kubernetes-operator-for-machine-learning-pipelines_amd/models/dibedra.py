"""Dibedra: a decoder of parallel layers for the serving runtime.

Layers are listed one by one in the configuration.  A layer's attention and its feed-forward read one normed
input and are added to one fp32 residual together; norms are dynamic tanh (no statistics).  Attention is
windowed, its queries and keys normed per head, its values the keys before norm and rotation, its output gated
per element.  The feed-forward is dense (tanh gelu), a mixture of experts, or absent:

  residual_begin | residual_step  ->  [k | gate | q | up] GEMM (gelu on the last columns)  ->  qk_head_norm (norm,
      rotation, paged stores)  ->  attention_hd into q's columns  ->  [O | down] GEMM  ->  residual_step
  experts beside it:  moe_dispatch_groups (router, choice, sort)  ->  grouped gate_up GEMM (clamped unit)  ->
      grouped down GEMM  ->  residual_step (sums a token's weighted expert rows, and its input for identity experts)

Both sublayers of a dense layer are two products: their input projections side by side, and their output
projections over the row [attention | gelu(up)].  In captured decode steps experts run beside attention.

A layer may use another's weights; every layer has pages of its own (``cache_layout``).

Weights are random-initialised on device, or read from a checkpoint while the model is built.  Rows and columns
are padded with zeros to whole GEMM tiles, so every size runs on the package's kernels.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F

from .. import ops
from ..parallel.comm import ParallelState, single
from ..runtime.kv_cache import KVLayer, pad_dim
from .config import AttentionSpec, DibedraConfig
from .layers import ParamSource, fuse_rows, linear, pad_to, rotary_table

GLU_ALPHA = 1.702  # of the experts' gated unit
MAX_OUTPUTS, MAX_TOP = 256, 64  # of the routing kernels
# captured decode steps of so many tokens run a layer's experts beside its attention, on a stream of their own.  (One
# token: joining the branches costs more than they gain.  Above 256 rows dense products may use the scratch that
# the experts' products share; captured steps are the only ones where the two run at once.)
SIDE_TOKENS = range(4, 257)


def _up(n: int, m: int) -> int:
    return -(-n // m) * m


class DibedraModel:
    def __init__(self, cfg: DibedraConfig, device="cuda", dtype=torch.bfloat16, pstate: ParallelState | None = None,
                 seed: int = 0, weights=None):
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.ps = pstate or single()
        if self.ps.tp.size > 1 or self.ps.ep.size > 1:
            raise ValueError("Dibedra runs on one GPU (no tensor / expert parallel form)")
        W = cfg.hidden_size
        self.width = pad_dim(W)  # of every row as stored
        src = ParamSource(weights, self.device, dtype, seed * 1000)
        self.embed = pad_to(src("embed", cfg.vocab_size, W), cfg.vocab_size, self.width)
        self.weights = {}  # by the layer that holds them
        self.cache_layout, self.state_shapes = [], []
        self._tables, self._table_len = {}, 0
        # decode work units per token: kv heads x groups of 16 query heads
        self.n_kv, self.v_pad = 1, 64
        for i, la in enumerate(cfg.layers):
            m = la.mixer
            if not isinstance(m, AttentionSpec) or not (m.tied_kv and m.head_norm and m.gate_elem) or m.sink or m.v_mix:
                raise ValueError(f"layer {i}: Dibedra has no such mixer ({m})")
            if la.moe and (la.moe.outputs > MAX_OUTPUTS or la.moe.top > MAX_TOP):
                raise ValueError(f"layer {i}: at most {MAX_OUTPUTS} router outputs, {MAX_TOP} of them per token")
            root = i if la.weights_of < 0 else la.weights_of
            if root not in self.weights:
                self.weights[root] = self._init_layer(src, f"l{root}.", cfg.layers[root])
            self.cache_layout.append(KVLayer(m.kv_heads, pad_dim(m.dim), pad_dim(m.dim)))
            self._tables.setdefault(m.rot, None)
            self.n_kv = max(self.n_kv, m.kv_heads * -(-(m.heads // m.kv_heads) // 16))
            self.v_pad = max(self.v_pad, pad_dim(m.dim))
        self.layers = [self.weights[i if la.weights_of < 0 else la.weights_of] for i, la in enumerate(cfg.layers)]
        # the logits' scale rides in the last norm
        alpha, w, b = self._norm(src, "final.norm")
        self.final_norm = (alpha, w * cfg.logit_scale, b * cfg.logit_scale)
        self.head = fuse_rows([pad_to(src("head", cfg.vocab_size, W), cfg.vocab_size, self.width)])
        # decode graphs only where every product is a kernel of this package: a library product may
        # record memory-set nodes, which have replayed wrongly
        ws = [self.head] + [L[k] for L in self.weights.values() for k in ("proj", "out")]
        self.graph_safe = dtype == torch.bfloat16 and all(ops.gemm_is_native(*w.shape) for w in ws)
        self.n_q = self.n_kv
        self._side = torch.cuda.Stream(self.device) if self.device.type == "cuda" else None
        # step metadata: one decode tile per one-token row, 128-token prompt tiles for every longer portion
        self.meta_kwargs = {"group": 16, "flash_tile": 128, "flash_min_q": 2, "part_dim": self.v_pad, "chunk": 0}

    # ------------------------------------------------------------- weights --
    def _norm(self, src, name):
        W, f32 = self.cfg.hidden_size, torch.float32
        pad = lambda t: F.pad(t, (0, self.width - W))  # noqa: E731  (zero columns stay zero)
        return (src(name + ".alpha", dtype=f32, mean=0.5, std=0.0).reshape(1),
                pad(src(name, W, dtype=f32, mean=1.0, std=0.0)), pad(src(name + ".b", W, dtype=f32, std=0.0)))

    def _init_layer(self, src, p, la):
        W, Wp, m = self.cfg.hidden_size, self.width, la.mixer
        nk, nq = m.kv_heads * m.dim, m.heads * m.dim
        # columns of the fused projection, each part on its own grid: keys, gates, then (one row of the output
        # product) queries, where attention leaves its result, and the dense feed-forward's columns
        g0 = _up(nk, 8)
        q0 = _up(g0 + nq, 64)
        u0 = _up(q0 + nq, 128) if la.ff else _up(q0 + nq, 64)
        end = u0 + _up(la.ff, 64)
        N = _up(end, 256) if end >= 2048 else end
        proj = torch.zeros(N, Wp, device=self.device, dtype=self.dtype)
        out = torch.zeros(Wp, end - q0, device=self.device, dtype=self.dtype)
        for at, n, name in ((0, nk, "mix.k"), (g0, nq, "mix.g"), (q0, nq, "mix.q"), (u0, la.ff, "mlp.up")):
            if n:
                proj[at:at + n, :W] = src(p + name, n, W)
        out[:W, :nq] = src(p + "mix.o", W, nq)
        if la.ff:
            out[:W, u0 - q0:u0 - q0 + la.ff] = src(p + "mlp.down", W, la.ff)
        L = {"proj": proj, "out": out, "g0": g0, "q0": q0, "u0": u0, "end": end, "norm": self._norm(src, p + "norm1"),
             **{f"{a}_norm": src(f"{p}mix.{a}.norm", m.dim, dtype=torch.float32, mean=1.0, std=0.0) for a in "qk"}}
        if la.moe:
            L.update(self._init_experts(src, p + "mlp.", la.moe))
        return L

    def _init_experts(self, src, p, m):
        W, Wp, fp = self.cfg.hidden_size, self.width, pad_dim(m.ff)
        L = {"w13": torch.empty(m.experts, 2 * fp, Wp, device=self.device, dtype=self.dtype),
             "w2": torch.empty(m.experts, Wp, fp, device=self.device, dtype=self.dtype)}
        for e in range(m.experts):
            gate, up = (pad_to(src(f"{p}e{e}.{n}", m.ff, W), fp, Wp) for n in ("gate", "up"))
            L["w13"][e] = ops.interleave_gate_up(gate, up)
            L["w2"][e] = pad_to(src(f"{p}e{e}.down", W, m.ff), Wp, fp)
        L["router"] = pad_to(src(p + "router", m.outputs, W), m.outputs, Wp)
        L["correction"] = src(p + "correction", m.outputs, dtype=torch.float32, std=0.0)
        return L

    def reserve_positions(self, n: int) -> None:
        """Rotary tables for positions below ``n`` (the engine's longest sequence)."""
        if n > self._table_len:
            self._tables = {rot: rotary_table(rot, n, device=self.device) for rot in self._tables}
            self._table_len = n

    # ---------------------------------------------------------- sublayers --
    def _layer(self, i, x, meta, kv):
        """Arguments of residual_step: what the layer's sublayers add."""
        L, la = self.layers[i], self.cfg.layers[i]
        m, eps = la.mixer, self.cfg.rms_eps
        k_cache, v_cache = kv.k[i], kv.v[i]
        g0, q0, nq = L["g0"], L["q0"], m.heads * m.dim
        side, experts = None, {}
        if la.moe and x.is_cuda and x.shape[0] in SIDE_TOKENS and torch.cuda.is_current_stream_capturing():
            side = self._side
            side.wait_stream(torch.cuda.current_stream())
            with torch.cuda.stream(side):
                experts = self._experts(L, la.moe, x)
        elif la.moe:
            experts = self._experts(L, la.moe, x)
        proj = ops.gemm(x, L["proj"], epi=ops.EPI_GELU, act_from=L["u0"]) if la.ff else linear(x, L["proj"])
        heads = proj[:, q0:q0 + nq]
        q = ops.qk_head_norm(heads, proj[:, :m.kv_heads * m.dim], None, m.heads, m.dim, m.vdim, L["q_norm"], L["k_norm"], eps,
                             self._tables[m.rot], meta.positions, meta.slots, k_cache, v_cache)
        # the heads' outputs take the queries' place
        ops.attention_hd(q, k_cache, v_cache, meta, m.dim, m.vdim, m.scale, gate=proj[:, g0:g0 + nq], window=m.window,
                         out=heads.unflatten(1, (m.heads, m.dim)))
        y = linear(proj[:, q0:L["end"]], L["out"])
        if side is not None:
            torch.cuda.current_stream().wait_stream(side)
        return {"y": y, **experts}

    def _experts(self, L, m, x):
        d = ops.moe_dispatch_groups(x, L["router"], L["correction"], m.experts, m.top, m.groups, m.keep)
        avg = max(1, x.shape[0] * m.top // m.outputs)
        a = ops.grouped_gemm(d.x, L["w13"], d.offsets, epi=ops.EPI_SILU_MUL, avg_rows=avg, a_rows=d.a_rows, glu=(GLU_ALPHA, m.limit))
        rows = ops.grouped_gemm(a, L["w2"], d.offsets, avg_rows=avg)
        return {"experts": (rows, d.inv, None), "share": (d.top_w, x if m.identity else None, d.self_w)}

    # ------------------------------------------------------------ forward --
    def forward(self, ids: torch.Tensor, meta, kv) -> torch.Tensor:
        """ids [T] int64; meta: AttnMeta; kv: KVCache with this model's layout.
        Returns the final-normed hidden states of every token times the logits' scale, [T, padded width]."""
        norms = [L["norm"] for L in self.layers] + [self.final_norm]
        alpha, w, b = norms[0]
        res, x = ops.residual_begin(ids, self.embed, 1.0, None, meta.positions, w, 0.0, tanh=(alpha, b))
        for i in range(len(self.layers)):
            alpha, w, b = norms[i + 1]
            x = ops.residual_step(res, post_w=None, norm_w=w, eps=0.0, store=i + 1 < len(self.layers), tanh=(alpha, b),
                                  **self._layer(i, x, meta, kv))
        return x

    def logits_local(self, hidden: torch.Tensor) -> torch.Tensor:
        """[n, padded width] -> logits [n, vocab] (model dtype)."""
        return linear(hidden, self.head)[:, :self.cfg.vocab_size]

    logits = logits_local

    def weight_tensors(self):
        yield self.embed
        for L in self.weights.values():
            for v in L.values():
                yield from (t for t in (v if isinstance(v, tuple) else (v,)) if isinstance(t, torch.Tensor))
        yield from self.final_norm
        yield self.head

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.weight_tensors())
