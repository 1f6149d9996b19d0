"""Kosesun: a hybrid decoder for the serving runtime.

Layers are listed one by one in the configuration; each has a mixer (softmax attention, or gated
linear attention) and possibly a squared-relu feed-forward, on hyper-connection streams:

  hyper_begin | hyper_step  ->  fused projection GEMM  ->
      attention: qk_norm_rope (q / k norm, rotary, value mixing, paged stores) -> attention_hd (sink,
                 output gate)
      gla:       gla (decay, recurrence, head norm, output gate)
  ->  O GEMM  ->  hyper_step  ->  up GEMM (relu^2 epilogue)  ->  down GEMM  ->  hyper_step ...

``hyper_step`` is this design's add + norm: it mixes the fp32 streams, adds the sublayer's output
and leaves the next sublayer's normed input, in one pass.  Attention layers keep keys and values in
the engine's paged cache (``cache_layout``), recurrent ones a state per sequence in its state slots
(``state_shapes``); the engine's scheduler, graphs and sampler run it like every other model.

Weights are random-initialised on device, or read from a checkpoint while the model is built.
"""
from __future__ import annotations

import torch

from .. import ops
from ..parallel.comm import ParallelState, single
from ..runtime.kv_cache import KVLayer, pad_dim
from .config import AttentionSpec, KosesunConfig
from .layers import ParamSource, fuse_rows, linear, rope_table

GLA_CHUNK = 64  # tokens of a recurrent layer's parallel prompt chunk (twice that in large steps)


class KosesunModel:
    def __init__(self, cfg: KosesunConfig, device="cuda", dtype=torch.bfloat16, pstate: ParallelState | None = None,
                 seed: int = 0, weights=None):
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.ps = pstate or single()
        if self.ps.tp.size > 1 or self.ps.ep.size > 1:
            raise ValueError("Kosesun runs on one GPU (no tensor / expert parallel form)")
        W, S = cfg.hidden_size, cfg.streams
        src = ParamSource(weights, self.device, dtype, seed * 1000)
        f32 = torch.float32
        self.embed = src("embed", cfg.vocab_size, W)
        self.layers, self.cache_layout, self.state_shapes = [], [], []
        self._rope_spec, self._rope, self._rope_len = set(), {}, 0
        # attention layers' decode work units per token: kv heads x groups of 16 query heads
        self.n_kv, self.v_pad = 1, 64
        subs = []  # sublayers in order: (run, streams' weights, norm)
        first_mix = None
        for i, la in enumerate(cfg.layers):
            p, m, L = f"l{i}.", la.mixer, {}
            proj = lambda *names: fuse_rows([src(f"{p}mix.{n}", rows, W) for n, rows in names])  # noqa: E731
            if isinstance(m, AttentionSpec):
                hq, hk, hv = m.heads * m.dim, m.kv_heads * m.dim, m.kv_heads * m.vdim
                L.update(proj=proj(("q", hq), ("k", hk), ("v", hv), ("g", m.heads)),
                         o=src(p + "mix.o", W, m.heads * m.vdim),
                         q_norm=src(p + "mix.q.norm", hq, dtype=f32, mean=1.0, std=0.0),
                         k_norm=src(p + "mix.k.norm", hk, dtype=f32, mean=1.0, std=0.0),
                         sink=src(p + "mix.sink", m.heads, dtype=f32, std=1.0), lam=None, cache=len(self.cache_layout))
                if m.v_mix and first_mix is None:
                    first_mix = m
                elif m.v_mix:
                    if m.kv_heads * m.vdim != first_mix.kv_heads * first_mix.vdim:
                        raise ValueError(f"layer {i}: value mixing needs the first mixing layer's value size")
                    L["lam"] = src(p + "mix.vmix", dtype=f32, mean=0.5, std=0.0).reshape(1)
                self.cache_layout.append(KVLayer(m.kv_heads, pad_dim(m.dim), pad_dim(m.vdim)))
                self._rope_spec.add((m.rot_base, m.rot_dims))
                self.n_kv = max(self.n_kv, m.kv_heads * -(-(m.heads // m.kv_heads) // 16))
                self.v_pad = max(self.v_pad, pad_dim(m.vdim))
                run = self._attention
            else:
                hk, hv = m.heads * m.dim, m.heads * m.vdim
                L.update(proj=proj(("q", hk), ("k", hk), ("v", hv), ("g", hv), ("a1", m.rank)),
                         o=src(p + "mix.o", W, hv), a2=src(p + "mix.a2", hk, m.rank),
                         a2_b=src(p + "mix.a2.b", hk, dtype=f32, mean=2.0, std=0.5),
                         norm=src(p + "mix.norm", m.vdim, dtype=f32, mean=1.0, std=0.0), state=len(self.state_shapes))
                self.state_shapes.append((m.heads, m.dim, m.vdim))
                run = self._gla
            self.layers.append(L)
            subs.append((run, i, self._streams(src, p + "hc1.", S), self._norm(src, p + "norm1", W)))
            if la.ff:
                L.update(up=src(p + "mlp.up", la.ff, W), down=src(p + "mlp.down", W, la.ff))
                subs.append((self._mlp, i, self._streams(src, p + "hc2.", S), self._norm(src, p + "norm2", W)))
        self.final_norm = self._norm(src, "final.norm", W)
        self.head = fuse_rows([src("head", cfg.vocab_size, W)])  # (padding rows: the logits rows stay 16-B aligned)
        self.ones = torch.ones(S, device=self.device, dtype=f32)
        self.subs = subs
        # decode graphs only where every product is a kernel of this package: a library product may
        # record memory-set nodes, which have replayed wrongly
        ws = [self.head] + [L[k] for L in self.layers for k in ("proj", "o", "up", "down") if k in L]
        self.graph_safe = dtype == torch.bfloat16 and all(ops.gemm_is_native(*w.shape) for w in ws)
        self.n_q = self.n_kv
        # step metadata: one decode tile per one-token row, 128-token prompt tiles for every longer
        # portion (both independent of a layer's head counts), chunks for the recurrent layers
        self.meta_kwargs = {"group": 16, "flash_tile": 128, "flash_min_q": 2, "part_dim": self.v_pad,
                            "chunk": GLA_CHUNK if self.state_shapes else 0}

    def _streams(self, src, p, S):
        f32 = torch.float32
        mix = src(p + "mix", S, S, dtype=f32, std=0.0)
        if src.w is None:
            mix.copy_(torch.eye(S, device=self.device))
        return {"in": src(p + "in", S, dtype=f32, mean=1.0 / S, std=0.0),
                "out": src(p + "out", S, dtype=f32, mean=1.0, std=0.0), "mix": mix}

    def _norm(self, src, name, n):
        return 1.0 + src(name, n, dtype=torch.float32, std=0.0)  # stored around zero

    def reserve_positions(self, n: int) -> None:
        """Rotary tables for positions below ``n`` (the engine's longest sequence)."""
        if n > self._rope_len:
            self._rope = {k: rope_table(k[1], n, k[0], device=self.device) for k in self._rope_spec}
            self._rope_len = n

    # ---------------------------------------------------------- sublayers --
    def _attention(self, i, x, meta, kv, ctx):
        L, m = self.layers[i], self.cfg.layers[i].mixer
        k, v = kv.k[L["cache"]], kv.v[L["cache"]]
        proj = linear(x, L["proj"])
        nq, nk, nv = m.heads * m.dim, m.kv_heads * m.dim, m.kv_heads * m.vdim
        values = proj[:, nq + nk:nq + nk + nv]
        if m.v_mix and "v_first" not in ctx:
            ctx["v_first"] = values
        q = ops.qk_norm_rope(proj, m.heads, m.dim, m.vdim, L["q_norm"], L["k_norm"], self.cfg.rms_eps,
                             self._rope[(m.rot_base, m.rot_dims)], meta.positions, meta.slots, k, v,
                             v_first=ctx["v_first"] if L["lam"] is not None else None, lam=L["lam"])
        gate = proj[:, nq + nk + nv:nq + nk + nv + m.heads]
        a = ops.attention_hd(q, k, v, meta, m.dim, m.vdim, m.scale, sink=L["sink"], gate=gate)
        return linear(a.view(a.shape[0], -1), L["o"])

    def _gla(self, i, x, meta, kv, ctx):
        L, m = self.layers[i], self.cfg.layers[i].mixer
        o = ops.gla(linear(x, L["proj"]), m.heads, m.dim, m.vdim, L["a2"], L["a2_b"], L["norm"], m.tau,
                    self.cfg.rms_eps, kv.states[L["state"]], meta)
        return linear(o, L["o"])

    def _mlp(self, i, x, meta, kv, ctx):
        L = self.layers[i]
        return linear(ops.gemm(x, L["up"], epi=ops.EPI_RELU2), L["down"])

    # ------------------------------------------------------------ forward --
    def forward(self, ids: torch.Tensor, meta, kv) -> torch.Tensor:
        """ids [T] int64; meta: AttnMeta; kv: KVCache with this model's layout and states.
        Returns the final-normed hidden states of every token [T, W]."""
        eps, ctx = self.cfg.rms_eps, {}
        _, _, hc, norm = self.subs[0]
        streams, x = ops.hyper_begin(ids, self.embed, self.cfg.embed_scale, self.cfg.streams, hc["in"], norm, eps)
        for n, (run, i, hc, _) in enumerate(self.subs):
            last = n + 1 == len(self.subs)
            nxt_in, nxt_norm = (self.ones, self.final_norm) if last else (self.subs[n + 1][2]["in"], self.subs[n + 1][3])
            x = ops.hyper_step(streams, run(i, x, meta, kv, ctx), hc["mix"], hc["out"], nxt_in, nxt_norm, eps,
                               store=not last)
        return x

    def logits_local(self, hidden: torch.Tensor) -> torch.Tensor:
        """[n, W] -> soft-capped logits [n, vocab] in fp32."""
        return ops.softcap(linear(hidden, self.head), self.cfg.logit_softcap)[:, :self.cfg.vocab_size]

    logits = logits_local

    def weight_tensors(self):
        yield self.embed
        for L in self.layers:
            yield from (v for v in L.values() if isinstance(v, torch.Tensor))
        for _, _, hc, norm in self.subs:
            yield from hc.values()
            yield norm
        yield self.final_norm
        yield self.head

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.weight_tensors())
