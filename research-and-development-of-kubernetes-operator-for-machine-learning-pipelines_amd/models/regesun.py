"""Regesun: a hybrid decoder for the serving runtime.

Layers are listed one by one in the configuration; each has a mixer (windowed latent attention,
selective state space, or the generalized delta rule) and possibly a clamped gated feed-forward, on one
fp32 residual stream with a norm before and behind every sublayer:

  residual_begin (embedding + learned position) | residual_step  ->  fused projection GEMM  ->
      latent attention: latent_store -> latent_attention (window, sink, output gate)
      state space:      short_conv -> ssd -> gated_norm (gate first, groups)
      delta rule:       delta (decay, removal, recurrence) -> gated_norm (per head, gate behind)
  ->  O GEMM  ->  residual_step  ->  gate_up GEMM (clamped unit in the epilogue)  ->  down GEMM  ->  ...

``residual_step`` norms the sublayer's output, adds it with the layer scale and leaves the next
sublayer's normed input, in one pass.  Attention layers keep one latent row per token in the engine's
paged cache (``cache_layout``), recurrent ones their state (and the convolution's last inputs) in the
sequence's state slots (``state_shapes``); the engine's scheduler, graphs and sampler run it like every
other model.

Weights are random-initialised on device, or read from a checkpoint while the model is built.
"""
from __future__ import annotations

import math

import torch

from .. import ops
from ..parallel.comm import ParallelState, single
from ..runtime.kv_cache import KVLayer, pad_dim
from .config import DeltaSpec, LatentAttentionSpec, RegesunConfig, SSDSpec
from .layers import ParamSource, fuse_rows, linear, pad_rows

CHUNK = 64                         # granule of the recurrent layers' prompt lists
GLU_ALPHA = 1.702                  # of the feed-forward's gate
DELTA_DECAY = math.exp(-0.5)       # largest log decay of the delta rule
UNIT_EPS = 1e-6                    # in the delta rule's unit keys


class RegesunModel:
    def __init__(self, cfg: RegesunConfig, device="cuda", dtype=torch.bfloat16, pstate: ParallelState | None = None,
                 seed: int = 0, weights=None):
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.ps = pstate or single()
        if self.ps.tp.size > 1 or self.ps.ep.size > 1:
            raise ValueError("Regesun runs on one GPU (no tensor / expert parallel form)")
        W = cfg.hidden_size
        src = ParamSource(weights, self.device, dtype, seed * 1000)
        ones = lambda name, n: src(name, n, dtype=torch.float32, mean=1.0, std=0.0)  # noqa: E731
        self.embed = src("embed", cfg.vocab_size, W)
        self.pos = src("pos", cfg.max_position, W)
        self.layers, self.cache_layout, self.state_shapes = [], [], []
        # decode work units per token: groups of 16 heads; partials hold latents
        self.n_kv, self.part_dim, windows = 1, 64, []
        self.subs = subs = []  # sublayers in order: (run, layer, norm before, norm behind x layer scale)
        for i, la in enumerate(cfg.layers):
            p, m = f"l{i}.", la.mixer
            if isinstance(m, LatentAttentionSpec):
                L, run = self._init_latent(src, p + "mix.", m), self._latent
                windows.append(m.window)
            elif isinstance(m, SSDSpec):
                L, run = self._init_ssd(src, p + "mix.", m), self._ssd
            elif isinstance(m, DeltaSpec):
                L, run = self._init_delta(src, p + "mix.", m), self._delta
            else:
                raise ValueError(f"layer {i}: Regesun has no mixer {type(m).__name__}")
            self.layers.append(L)
            subs.append((run, i, ones(p + "norm1", W), ones(p + "norm1b", W) * ones(p + "ls1", W)))
            if la.ff:
                pad = -la.ff % 64  # zero rows of the gate and up projections, zero columns of down
                gate, up = (torch.nn.functional.pad(src(f"{p}mlp.{n}", la.ff, W), (0, 0, 0, pad)) for n in ("gate", "up"))
                L.update(gate_up=ops.interleave_gate_up(gate, up).contiguous(),
                         down=torch.nn.functional.pad(src(p + "mlp.down", W, la.ff), (0, pad)).contiguous())
                subs.append((self._mlp, i, ones(p + "norm2", W), ones(p + "norm2b", W) * ones(p + "ls2", W)))
        self.final_norm = ones("final.norm", W)
        self.head = fuse_rows([src("head", cfg.vocab_size, W)])
        # decode graphs only where every product is a kernel of this package: a library product may
        # record memory-set nodes, which have replayed wrongly
        ws = [self.head] + [L[k] for L in self.layers for k in ("proj", "o", "gate_up", "down") if k in L]
        self.graph_safe = dtype == torch.bfloat16 and all(ops.gemm_is_native(*w.shape) for w in ws)
        self.n_q = self.n_kv
        # step metadata: one decode tile per one-token row, 128-token prompt tiles and chunks for every
        # longer portion
        self.meta_kwargs = {"group": 16, "flash_tile": 128, "flash_min_q": 2, "part_dim": self.part_dim, "chunk": CHUNK,
                            "expand_window": (0 if 0 in windows else max(windows)) if windows else None}

    # ------------------------------------------------------------- weights --
    def _init_latent(self, src, p, m):
        W, H, R = self.cfg.hidden_size, m.heads, m.rank
        KP, VP, RP = pad_dim(m.dim), pad_dim(m.vdim), pad_dim(R)
        uk, uv = src(p + "uk", H * m.dim, R), src(p + "uv", H * m.vdim, R)
        pad_r = lambda w: torch.nn.functional.pad(w, (0, RP - R))  # noqa: E731
        # a head's query rows and the latent's rows padded to the kernels' row sizes with zeros
        L = {"proj": fuse_rows([pad_rows(src(p + "q", H * m.dim, W), H, KP), pad_rows(src(p + "dkv", R, W), 1, RP),
                                src(p + "g", H * m.vdim, W)]),
             "c_norm": src(p + "dkv.norm", R, dtype=torch.float32, mean=1.0, std=0.0),
             "w_kv": pad_r(torch.cat([pad_rows(uk, H, KP), pad_rows(uv, H, VP)])).contiguous(),
             "w_qk": torch.nn.functional.pad(uk.view(H, m.dim, R).transpose(1, 2), (0, KP - m.dim, 0, RP - R)).contiguous(),
             "w_vo": pad_r(uv.view(H, m.vdim, R)).contiguous(),
             "sink": src(p + "sink", H, dtype=torch.float32, std=1.0), "o": src(p + "o", W, H * m.vdim),
             "cache": len(self.cache_layout)}
        self.cache_layout.append(KVLayer(1, RP, 0))
        self.n_kv, self.part_dim = max(self.n_kv, -(-H // 16)), max(self.part_dim, RP)
        return L

    def _init_ssd(self, src, p, m):
        W, f32 = self.cfg.hidden_size, torch.float32
        L = {"proj": fuse_rows([src(p + "in", 2 * m.inner + 2 * m.groups * m.state + m.heads, W)]),
             "conv": src(p + "conv", m.channels, m.taps, dtype=f32, std=0.3), "conv_b": src(p + "conv.b", m.channels, dtype=f32),
             "dt_bias": src(p + "dt_bias", m.heads, dtype=f32, mean=-3.0, std=1.0),
             "a_neg": -torch.exp(src(p + "A_log", m.heads, dtype=f32, mean=1.0, std=0.7)),
             "d_skip": src(p + "D", m.heads, dtype=f32, mean=1.0, std=0.0),
             "norm": src(p + "norm", m.inner, dtype=f32, mean=1.0, std=0.0), "o": src(p + "o", W, m.inner),
             "tail": len(self.state_shapes), "state": len(self.state_shapes) + 1}
        self.state_shapes += [(m.taps - 1, m.channels), (m.heads, m.state, m.vdim)]
        return L

    def _init_delta(self, src, p, m):
        W, f32, n = self.cfg.hidden_size, torch.float32, m.heads * m.dim
        L = {"proj": fuse_rows([*(src(p + k, n, W) for k in "rkva"), src(p + "w1", m.rank, W), src(p + "g", n, W)]),
             "w2": src(p + "w2", n, m.rank), "w0": src(p + "w0", n, dtype=f32, mean=-2.0, std=1.0),
             "a_b": src(p + "a.b", n, dtype=f32, std=1.0), "norm": src(p + "norm", n, dtype=f32, mean=1.0, std=0.0),
             "o": src(p + "o", W, n), "state": len(self.state_shapes)}
        self.state_shapes.append((m.heads, m.dim, m.dim))
        return L

    # ---------------------------------------------------------- sublayers --
    def _latent(self, i, x, meta, kv):
        L, m = self.layers[i], self.cfg.layers[i].mixer
        cache, KP = kv.k[L["cache"]], pad_dim(m.dim)
        proj = linear(x, L["proj"])
        nq, nr = m.heads * KP, cache.shape[3]
        ops.latent_store(proj[:, nq:nq + m.rank], L["c_norm"], self.cfg.rms_eps, meta.slots, cache)
        o = ops.latent_attention(proj[:, :nq].unflatten(1, (m.heads, KP)), proj[:, nq + nr:nq + nr + m.heads * m.vdim],
                                 cache, L["w_kv"], L["w_qk"], L["w_vo"], m.vdim, m.scale, m.window, L["sink"], meta)
        return linear(o, L["o"])

    def _ssd(self, i, x, meta, kv):
        L, m = self.layers[i], self.cfg.layers[i].mixer
        proj = linear(x, L["proj"])
        n, c = m.inner, m.channels
        xbc = ops.short_conv(proj[:, n:n + c], L["conv"], L["conv_b"], kv.states[L["tail"]], meta)
        y = ops.ssd(xbc, proj[:, n + c:n + c + m.heads], m.groups, L["dt_bias"], L["a_neg"], L["d_skip"],
                    kv.states[L["state"]], meta)
        y = ops.gated_norm(y, proj[:, :n], L["norm"], m.norm_groups, self.cfg.rms_eps, "silu", gate_first=True)
        return linear(y, L["o"])

    def _delta(self, i, x, meta, kv):
        L, m = self.layers[i], self.cfg.layers[i].mixer
        proj = linear(x, L["proj"])
        n = m.heads * m.dim
        o = ops.delta(proj, L["w2"], L["w0"], L["a_b"], DELTA_DECAY, UNIT_EPS, kv.states[L["state"]], meta)
        g = 4 * n + m.rank
        o = ops.gated_norm(o, proj[:, g:g + n], L["norm"], m.heads, self.cfg.rms_eps, "sigmoid", gate_first=False)
        return linear(o, L["o"])

    def _mlp(self, i, x, meta, kv):
        L = self.layers[i]
        act = ops.gemm(x, L["gate_up"], epi=ops.EPI_SILU_MUL, glu=(GLU_ALPHA, self.cfg.layers[i].limit))
        return linear(act, L["down"])

    # ------------------------------------------------------------ forward --
    def forward(self, ids: torch.Tensor, meta, kv) -> torch.Tensor:
        """ids [T] int64; meta: AttnMeta; kv: KVCache with this model's layout and states.
        Returns the final-normed hidden states of every token [T, W]."""
        eps, subs = self.cfg.rms_eps, self.subs
        res, x = ops.residual_begin(ids, self.embed, 1.0, self.pos, meta.positions, subs[0][2], eps)
        for n, (run, i, _, post) in enumerate(subs):
            last = n + 1 == len(subs)
            x = ops.residual_step(res, run(i, x, meta, kv), post, self.final_norm if last else subs[n + 1][2], eps,
                                  store=not last)
        return x

    def logits_local(self, hidden: torch.Tensor) -> torch.Tensor:
        """[n, W] -> logits [n, vocab] (model dtype)."""
        return linear(hidden, self.head)[:, :self.cfg.vocab_size]

    logits = logits_local

    def weight_tensors(self):
        yield self.embed
        yield self.pos
        for L in self.layers:
            yield from (v for v in L.values() if isinstance(v, torch.Tensor))
        for _, _, norm, post in self.subs:
            yield norm
            yield post
        yield self.final_norm
        yield self.head

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.weight_tensors())
