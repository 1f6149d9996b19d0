"""Building blocks shared by the model families: GEMM entry point, RoPE tables,
random on-device weight init (G4: no host-side materialisation of 16-141 GB).
"""
from __future__ import annotations

import math

import torch
import torch.nn.functional as F

from .. import ops


def linear(x: torch.Tensor, w: torch.Tensor, out: torch.Tensor | None = None) -> torch.Tensor:
    """y = x @ w^T with w stored [N, K] (row-major out-features).

    Routed through ``ops.gemm`` which picks the hand-written MFMA kernel for
    the shapes it covers and hipBLASLt for the rest (plain library GEMM)."""
    return ops.gemm(x, w, out=out) if hasattr(ops, "gemm") else F.linear(x, w, out=out)


def rope_inv_freq(head_dim: int, theta: float, scaling: dict | None = None) -> torch.Tensor:
    inv = 1.0 / (theta ** (torch.arange(0, head_dim, 2, dtype=torch.float64) / head_dim))
    if scaling and scaling.get("rope_type", scaling.get("type")) == "llama3":
        factor = scaling.get("factor", 8.0)
        lo, hi = scaling.get("low_freq_factor", 1.0), scaling.get("high_freq_factor", 4.0)
        old = scaling.get("original_max_position_embeddings", 8192)
        lo_wl, hi_wl = old / lo, old / hi
        wl = 2 * math.pi / inv
        smooth = (old / wl - lo) / (hi - lo)
        scaled = torch.where(wl > lo_wl, inv / factor, inv)
        mid = (wl <= lo_wl) & (wl >= hi_wl)
        inv = torch.where(mid, (1 - smooth) * inv / factor + smooth * inv, scaled)
    return inv


def rope_table(head_dim: int, max_pos: int, theta: float, scaling: dict | None = None,
               device=None) -> torch.Tensor:
    """[max_pos, head_dim] fp32: cos in [:, :D/2], sin in [:, D/2:] (host-precomputed)."""
    inv = rope_inv_freq(head_dim, theta, scaling)
    t = torch.arange(max_pos, dtype=torch.float64)
    f = torch.outer(t, inv)
    return torch.cat([f.cos(), f.sin()], dim=-1).float().to(device)


def rotary_table(rot, max_pos: int, device=None) -> torch.Tensor:
    """[max_pos, dims] fp32 of a ``RotarySpec``: cos of the dims / 2 pairs, then sin (angles in fp64 on the
    host)."""
    inv, mult = rope_inv_freq(rot.dims, rot.base), 1.0
    if rot.scaling is not None:
        y = rot.scaling
        # the pair that turns t times in the original range
        pair = lambda t: rot.dims * math.log(y.original / (2 * math.pi * t)) / (2 * math.log(rot.base))  # noqa: E731
        lo, hi = max(math.floor(pair(y.fast)), 0), min(math.ceil(pair(y.slow)), rot.dims - 1)
        ramp = ((torch.arange(rot.dims // 2, dtype=torch.float64) - lo) / max(hi - lo, 1e-3)).clamp(0, 1)
        inv, mult = inv / y.factor * ramp + inv * (1 - ramp), 0.1 * math.log(y.factor) + 1
    f = torch.outer(torch.arange(max_pos, dtype=torch.float64), inv)
    return (torch.cat([f.cos(), f.sin()], dim=-1) * mult).float().to(device)


def pad_to(w: torch.Tensor, rows: int, cols: int) -> torch.Tensor:
    """[n, K] with zero rows and columns up to [rows, cols]."""
    return F.pad(w, (0, cols - w.shape[1], 0, rows - w.shape[0])).contiguous()


def pad_rows(w: torch.Tensor, heads: int, rows: int) -> torch.Tensor:
    """[heads * d, K] -> [heads * rows, K], every head's rows padded with zeros."""
    v = w.view(heads, -1, w.shape[1])
    return F.pad(v, (0, 0, 0, rows - v.shape[1])).reshape(heads * rows, w.shape[1])


def init_weight(shape, device, dtype=torch.bfloat16, std: float = 0.02, gen: torch.Generator | None = None):
    w = torch.empty(*shape, device=device, dtype=dtype)
    w.normal_(0.0, std, generator=gen)
    return w


def init_norm(n, device, dtype=torch.bfloat16):
    return torch.ones(n, device=device, dtype=dtype)


def fuse_rows(parts, multiple: int = 16, large: int = 256) -> torch.Tensor:
    """Projections of one input stacked into one weight [N, K], zero rows up to a whole number of
    GEMM tiles (``large`` from 2048 rows, where the 256-column tiles run)."""
    n = sum(p.shape[0] for p in parts)
    m = large if n >= 2048 else multiple
    pad = -n % m
    if pad:
        parts = [*parts, parts[0].new_zeros(pad, parts[0].shape[1])]
    return torch.cat(parts, 0).contiguous()


class ParamSource:
    """Tensors by name while a model is built: a checkpoint's, or random ones of the asked shape."""

    def __init__(self, weights, device, dtype, seed: int):
        self.w, self.device, self.dtype = weights, device, dtype
        self.gen = torch.Generator(device=device)
        self.gen.manual_seed(seed)

    def __call__(self, name: str, *shape, dtype=None, mean: float = 0.0, std: float = 0.02) -> torch.Tensor:
        dtype = dtype or self.dtype
        if self.w is None:
            t = torch.empty(shape, device=self.device, dtype=dtype)
            return t.normal_(mean, std, generator=self.gen) if std else t.fill_(mean)
        t = self.w.get(name)
        if tuple(t.shape) != shape:
            raise ValueError(f"checkpoint tensor {name!r} has shape {tuple(t.shape)}, expected {shape}")
        return t.to(self.device, dtype).contiguous()
