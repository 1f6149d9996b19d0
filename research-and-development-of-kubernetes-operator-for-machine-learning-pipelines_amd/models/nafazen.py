"""Nafazen: a decoder of latent-attention layers for the serving runtime.

Layers are listed one by one in the configuration.  Each has latent attention (queries through a latent of
their own, a rotated key part shared by all heads, the layer's latents its own or an earlier layer's) and
possibly a feed-forward, dense with the xIELU activation or a mixture of experts, on one fp32 residual
stream.  Norms stand behind the sublayers only, with one number for all coordinates:

  residual_begin | residual_step  ->  [query latent | latent | rotated key] GEMM  ->  latent_store (both norms,
      rotation, paged store)  ->  query GEMM  ->  latent_attention  ->  O GEMM  ->  residual_step
  dense:    up GEMM (xIELU epilogue)  ->  down GEMM  ->  residual_step
  experts:  moe_dispatch_input (router, choice, sort)  ->  grouped gate_up GEMM (rows times their scores)  ->
      grouped down GEMM, beside the shared expert's two  ->  residual_step (sums a token's expert rows)

``residual_step`` forms the sublayer's output, norms it and adds it, in one pass; sublayers read the residual
itself.  The engine keeps one row [latent | rotated key] per token and layer with latents of its own
(``cache_layout``).

Weights are random-initialised on device, or read from a checkpoint while the model is built.  Rows and columns
are padded with zeros to whole GEMM tiles, so every size runs on the package's kernels.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F

from .. import ops
from ..parallel.comm import ParallelState, single
from ..runtime.kv_cache import KVLayer, pad_dim
from .config import LatentAttentionSpec, NafazenConfig
from .layers import ParamSource, fuse_rows, linear, pad_rows, pad_to, rotary_table

CHUNK = 64  # granule of the step's list of prompt portions
MAX_EXPERTS, MAX_TOP = 256, 64  # of the routing kernels


def _up8(n: int) -> int:
    return -(-n // 8) * 8


class NafazenModel:
    def __init__(self, cfg: NafazenConfig, device="cuda", dtype=torch.bfloat16, pstate: ParallelState | None = None,
                 seed: int = 0, weights=None):
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.ps = pstate or single()
        if self.ps.tp.size > 1 or self.ps.ep.size > 1:
            raise ValueError("Nafazen runs on one GPU (no tensor / expert parallel form)")
        W = cfg.hidden_size
        self.width = pad_dim(W)  # of every row as stored
        src = ParamSource(weights, self.device, dtype, seed * 1000)
        number = lambda name: src(name, dtype=torch.float32, mean=1.0, std=0.0).reshape(1)  # noqa: E731
        self.embed = pad_to(src("embed", cfg.vocab_size, W), cfg.vocab_size, self.width)
        self.layers, self.cache_layout, self.state_shapes = [], [], []
        self._tables, self._table_len = {}, 0
        # decode work units per token: groups of 16 heads; partials hold latents
        self.n_kv, self.part_dim = 1, 64
        self.subs = subs = []  # sublayers in order: (run, layer, norm)
        for i, la in enumerate(cfg.layers):
            p = f"l{i}."
            if not isinstance(la.mixer, LatentAttentionSpec):
                raise ValueError(f"layer {i}: Nafazen has no mixer {type(la.mixer).__name__}")
            L = self._init_attention(src, p + "mix.", la.mixer)
            self.layers.append(L)
            subs.append((self._attention, i, number(p + "norm1")))
            if la.moe:
                if la.moe.experts > MAX_EXPERTS or la.moe.top > MAX_TOP:
                    raise ValueError(f"layer {i}: at most {MAX_EXPERTS} experts, {MAX_TOP} of them per token")
                L.update(self._init_experts(src, p + "mlp.", la.moe))
                subs.append((self._experts, i, number(p + "norm2")))
            elif la.ff:
                L.update(self._init_dense(src, p + "mlp.", la.ff))
                subs.append((self._dense, i, number(p + "norm2")))
        self.final_norm = number("final.norm")
        self.head = fuse_rows([pad_to(src("head", cfg.vocab_size, W), cfg.vocab_size, self.width)])
        # decode graphs only where every product is a kernel of this package: a library product may
        # record memory-set nodes, which have replayed wrongly
        ws = [self.head] + [v for L in self.layers for k, v in L.items() if k in ("down_q", "uq", "o", "up", "down", "s_gate_up",
                                                                                  "s_down")]
        self.graph_safe = dtype == torch.bfloat16 and all(ops.gemm_is_native(*w.shape) for w in ws)
        self.n_q = self.n_kv
        # step metadata: one decode tile per one-token row, 128-token prompt tiles for every longer portion,
        # whose keys are expanded (all of them: no windows)
        self.meta_kwargs = {"group": 16, "flash_tile": 128, "flash_min_q": 2, "part_dim": self.part_dim, "chunk": CHUNK,
                            "expand_window": 0}

    # ------------------------------------------------------------- weights --
    def _init_attention(self, src, p, m):
        W, Wp, H, R, rot = self.cfg.hidden_size, self.width, m.heads, m.rank, m.rot_dim
        # a head's query: [unrotated | rotated], a cached row: [latent | rotated key]; parts start on 8
        q_off, k_off, QP = _up8(m.dim), _up8(R), pad_dim(m.q_rank)
        KP, RP, KD = pad_dim(q_off + rot), pad_dim(k_off + rot), pad_dim(q_off)
        VH = _up8(m.vdim)
        while H * VH % 64:
            VH += 8
        down = [pad_to(src(p + "dq", m.q_rank, W), QP, Wp)]
        L = {"q_norm": src(p + "dq.norm", m.q_rank, dtype=torch.float32, mean=1.0, std=0.0), "QP": QP, "KP": KP, "VH": VH,
             "q_off": q_off, "k_off": k_off}
        if m.kv_from < 0:
            dkv = src(p + "dkv", R + rot, W)
            down += [pad_to(dkv[:R], k_off, Wp), pad_to(dkv[R:], rot, Wp)]
            L["c_norm"] = src(p + "dkv.norm", R, dtype=torch.float32, mean=1.0, std=0.0)
            L["cache"] = len(self.cache_layout)
            self.cache_layout.append(KVLayer(1, RP, 0))
        else:
            L["cache"] = self.layers[m.kv_from]["cache"]
        uq = src(p + "uq", H * (m.dim + rot), m.q_rank).view(H, m.dim + rot, m.q_rank)
        uq = torch.cat([F.pad(uq[:, :m.dim], (0, 0, 0, q_off - m.dim)), F.pad(uq[:, m.dim:], (0, 0, 0, KP - q_off - rot))], 1)
        uk, uv = src(p + "uk", H * m.dim, R), src(p + "uv", H * m.vdim, R)
        # expanding rows: a head's key is its map of the latent, then the row's rotated part as it is
        same = torch.zeros(H, KP, RP, device=self.device, dtype=self.dtype)
        same[:, :m.dim, :R] = uk.view(H, m.dim, R)
        same[:, q_off:q_off + rot, k_off:k_off + rot] = torch.eye(rot, device=self.device, dtype=self.dtype)
        L.update(down_q=fuse_rows(down), uq=pad_to(uq.reshape(H * KP, m.q_rank), H * KP, QP),
                 w_kv=torch.cat([same.view(H * KP, RP), pad_to(pad_rows(uv, H, pad_dim(VH)), H * pad_dim(VH), RP)]).contiguous(),
                 w_qk=F.pad(uk.view(H, m.dim, R).transpose(1, 2), (0, KD - m.dim, 0, k_off - R)).contiguous(),
                 w_vo=F.pad(uv.view(H, m.vdim, R), (0, pad_dim(R) - R, 0, VH - m.vdim)).contiguous(),
                 o=pad_to(F.pad(src(p + "o", W, H * m.vdim).view(W, H, m.vdim), (0, VH - m.vdim)).reshape(W, H * VH), Wp, H * VH))
        self._tables.setdefault(m.rot, None)
        self.n_kv, self.part_dim = max(self.n_kv, -(-H // 16)), max(self.part_dim, RP)
        return L

    def _init_dense(self, src, p, ff):
        W, Wp, fp = self.cfg.hidden_size, self.width, pad_dim(ff)
        a, b = F.softplus(src(p + "act", 2, dtype=torch.float32, std=0.5).double()).tolist()
        return {"up": pad_to(src(p + "up", ff, W), fp, Wp), "down": pad_to(src(p + "down", W, ff), Wp, fp), "act": (a, b + 0.5)}

    def _gated(self, src, p, ff):
        """(gate and up rows interleaved, down) of a gated feed-forward, in whole tiles."""
        W, Wp, fp = self.cfg.hidden_size, self.width, pad_dim(ff)
        gate, up = (pad_to(src(p + n, ff, W), fp, Wp) for n in ("gate", "up"))
        return ops.interleave_gate_up(gate, up).contiguous(), pad_to(src(p + "down", W, ff), Wp, fp)

    def _init_experts(self, src, p, m):
        W, Wp, fp = self.cfg.hidden_size, self.width, pad_dim(m.ff)
        L = {"w13": torch.empty(m.experts, 2 * fp, Wp, device=self.device, dtype=self.dtype),
             "w2": torch.empty(m.experts, Wp, fp, device=self.device, dtype=self.dtype)}
        for e in range(m.experts):
            L["w13"][e], L["w2"][e] = self._gated(src, f"{p}e{e}.", m.ff)
        router = [src(p + "router", m.experts, W)]
        if m.shared:
            L["s_gate_up"], L["s_down"] = self._gated(src, p + "shared.", m.shared)
            router.append(src(p + "shared.sg", 1, W))  # rides behind the router's rows
        L["router"] = pad_to(torch.cat(router), sum(r.shape[0] for r in router), Wp)
        return L

    def reserve_positions(self, n: int) -> None:
        """Rotary tables for positions below ``n`` (the engine's longest sequence)."""
        if n > self._table_len:
            self._tables = {rot: rotary_table(rot, n, device=self.device) for rot in self._tables}
            self._table_len = n

    # ---------------------------------------------------------- sublayers --
    def _attention(self, i, x, meta, kv):
        L, m = self.layers[i], self.cfg.layers[i].mixer
        cache, table, QP, k_off = kv.k[L["cache"]], self._tables[m.rot], L["QP"], L["k_off"]
        proj = linear(x, L["down_q"])
        query = (proj[:, :m.q_rank], L["q_norm"], QP)
        if m.kv_from < 0:
            rope = (proj[:, QP + k_off:QP + k_off + m.rot_dim], table, meta.positions, k_off)
            c_q = ops.latent_store(proj[:, QP:QP + m.rank], L["c_norm"], self.cfg.rms_eps, meta.slots, cache, rope, query)
        else:
            c_q = ops.latent_query(*query, self.cfg.rms_eps)
        q = linear(c_q, L["uq"]).unflatten(1, (m.heads, L["KP"]))
        o = ops.latent_attention(q, None, cache, L["w_kv"], L["w_qk"], L["w_vo"], L["VH"], m.scale, m.window, None, meta,
                                 rope=(table, m.rot_dim, L["q_off"], k_off))
        return {"y": linear(o, L["o"])}

    def _dense(self, i, x, meta, kv):
        L = self.layers[i]
        return {"y": linear(ops.gemm(x, L["up"], epi=ops.EPI_XIELU, xielu=L["act"]), L["down"])}

    def _experts(self, i, x, meta, kv):
        L, m = self.layers[i], self.cfg.layers[i].moe
        d = ops.moe_dispatch_input(x, L["router"], m.experts, m.top)
        avg = max(1, x.shape[0] * m.top // m.experts)
        a = ops.grouped_gemm(d.x, L["w13"], d.offsets, epi=ops.EPI_SILU_MUL, avg_rows=avg, a_rows=d.a_rows, row_scale=d.row_w)
        rows = ops.grouped_gemm(a, L["w2"], d.offsets, avg_rows=avg)
        y = linear(ops.gemm(x, L["s_gate_up"], epi=ops.EPI_SILU_MUL), L["s_down"]) if m.shared else None
        return {"y": y, "experts": (rows, d.inv, d.gate)}

    # ------------------------------------------------------------ forward --
    def forward(self, ids: torch.Tensor, meta, kv) -> torch.Tensor:
        """ids [T] int64; meta: AttnMeta; kv: KVCache with this model's layout.
        Returns the final-normed hidden states of every token, [T, padded width]."""
        cfg, eps, W = self.cfg, self.cfg.rms_eps, self.cfg.hidden_size
        res, x = ops.residual_begin(ids, self.embed, cfg.embed_scale, None, meta.positions, None, eps, width=W)
        for n, (run, i, norm) in enumerate(self.subs):
            last = n + 1 == len(self.subs)
            x = ops.residual_step(res, post_w=norm, norm_w=self.final_norm if last else None, eps=eps, store=not last, width=W,
                                  **run(i, x, meta, kv))
        return x

    def logits_local(self, hidden: torch.Tensor) -> torch.Tensor:
        """[n, padded width] -> logits [n, vocab], soft-capped in fp32 (no cap: as the product leaves them)."""
        lg = linear(hidden, self.head)
        return (ops.softcap(lg, self.cfg.logit_softcap) if self.cfg.logit_softcap else lg)[:, :self.cfg.vocab_size]

    logits = logits_local

    def weight_tensors(self):
        yield self.embed
        for L in self.layers:
            yield from (v for v in L.values() if isinstance(v, torch.Tensor))
        for _, _, norm in self.subs:
            yield norm
        yield self.final_norm
        yield self.head

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.weight_tensors())
