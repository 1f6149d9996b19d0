"""Plain, slow implementation of the Nafazen decoder, the oracle of its tests.

One function per mechanism, whole sequences, no cache, no batching.  It works on a checkpoint as it is
stored (the config.json dictionary and the tensors by name) in float64 by default, and shares no code
with the package under test.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x divided by its root mean square over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def scalar_norm(x, g, eps):
    """Norm with one number for all coordinates."""
    return rms(x, eps) * g


def yarn_ramp(n_pairs, base, dims, original, fast, slow):
    """Share of the stretched frequency per pair."""
    dim_of = lambda turns: dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))  # noqa: E731
    lo, hi = max(math.floor(dim_of(fast)), 0), min(math.ceil(dim_of(slow)), dims - 1)
    return [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(n_pairs)]


def frequencies(rot):
    """Angle per position of every pair, and the factor on cos and sin."""
    f = [rot["base"] ** (-2 * i / rot["dims"]) for i in range(rot["dims"] // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    ramp = yarn_ramp(len(f), rot["base"], rot["dims"], sc["original"], sc["fast"], sc["slow"])
    return [a / sc["factor"] * r + a * (1 - r) for a, r in zip(f, ramp)], 0.1 * math.log(sc["factor"]) + 1


def rotate(x, rot, pos0=0):
    """x [T, heads, D] at positions pos0, pos0 + 1, ..: pairs (2i, 2i + 1) of the first dims turn."""
    out = x.clone()
    freqs, mult = frequencies(rot)
    pos = torch.arange(pos0, pos0 + x.shape[0], dtype=x.dtype)
    for i, f in enumerate(freqs):
        c, s = (torch.cos(pos * f) * mult)[:, None], (torch.sin(pos * f) * mult)[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i], out[:, :, 2 * i + 1] = u * c - v * s, v * c + u * s
    return out


def causal_attention(q, k, v, q_rot, k_rot, scale):
    """q, k [T, H, D] and the rotated parts q_rot [T, H, R], k_rot [T, R] (one for all heads), v [T, H, V]."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        for h in range(H):
            s = (k[:i + 1, h] @ q[i, h] + k_rot[:i + 1] @ q_rot[i, h]) * scale
            e = torch.exp(s - s.max())
            out[i, h] = (e / e.sum()) @ v[:i + 1, h]
    return out


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + z.clamp(min=0)


def xielu(z, p, q):
    pos = softplus(p) * z * z + z / 2
    neg = (0.5 + softplus(q)) * (torch.expm1(z.clamp(max=0)) - z) + z / 2
    return torch.where(z > 0, pos, neg)


def silu(z):
    return z * torch.sigmoid(z)


def gated_ff(x, gate, up, down):
    return (silu(x @ gate.T) * (x @ up.T)) @ down.T


def choose(z, top):
    """Router logits of one token -> [(expert, weight)]."""
    s = torch.sigmoid(z)
    best = torch.argsort(s, descending=True)[:top]
    return [(int(e), s[e]) for e in best]


def shared_gate(z):
    return torch.sigmoid(z)


def weighted_expert(ff, h, w):
    """The weight is on the expert's input."""
    return ff(w * h)


def softcap(x, cap):
    return cap * torch.tanh(x / cap)


class Oracle:
    """``cfg``: config.json as a dictionary, ``weights``: name -> tensor."""

    def __init__(self, cfg, weights, dtype=torch.float64):
        self.cfg = cfg
        self.w = {k: v.to(dtype) for k, v in weights.items()}
        self.eps = cfg["norm"]["eps"]

    def latent(self, p, m, h):
        """(normed latent, rotated shared key) of every token: what a layer caches."""
        w, R = self.w, m["kv_rank"]
        d = h @ w[p + "dkv"].T
        return rms(d[:, :R], self.eps) * w[p + "dkv.norm"], rotate(d[:, None, R:], m["rot"])[:, 0]

    def attention(self, p, m, h, ctx):
        w, T, H, D = self.w, h.shape[0], m["heads"], m["dim"]
        c_q = rms(h @ w[p + "dq"].T, self.eps) * w[p + "dq.norm"]
        q = (c_q @ w[p + "uq"].T).view(T, H, D + m["rot_dim"])
        ctx[p] = c, k_rot = ctx[f"l{m['kv_from']}.mix."] if "kv_from" in m else self.latent(p, m, h)
        k, v = (c @ w[p + "uk"].T).view(T, H, D), (c @ w[p + "uv"].T).view(T, H, m["vdim"])
        o = causal_attention(q[..., :D], k, v, rotate(q[..., D:], m["rot"]), k_rot, m["scale"])
        return o.reshape(T, H * m["vdim"]) @ w[p + "o"].T

    def dense(self, p, m, h):
        w = self.w
        return xielu(h @ w[p + "up"].T, w[p + "act"][0], w[p + "act"][1]) @ w[p + "down"].T

    def moe(self, p, m, h):
        w = self.w
        ff = lambda q: lambda x: gated_ff(x, w[q + "gate"], w[q + "up"], w[q + "down"])  # noqa: E731
        out = shared_gate(h @ w[p + "shared.sg"].T) * ff(p + "shared.")(h)
        z = h @ w[p + "router"].T
        for t in range(h.shape[0]):
            for e, s in choose(z[t], m["router"]["top"]):
                out[t] += weighted_expert(ff(f"{p}e{e}."), h[t], s)
        return out

    def run(self, tokens):
        """(logits [T, vocab], [residual after every layer])."""
        cfg, w, eps, ctx = self.cfg, self.w, self.eps, {}
        x = w["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
        after = []
        for i, lay in enumerate(cfg["layers"]):
            p = f"l{i}."
            x = x + scalar_norm(self.attention(p + "mix.", lay["mixer"], x, ctx), w[p + "norm1"], eps)
            if lay.get("mlp"):
                ff = {"dense": self.dense, "moe": self.moe}[lay["mlp"]["kind"]]
                x = x + scalar_norm(ff(p + "mlp.", lay["mlp"], x), w[p + "norm2"], eps)
            after.append(x)
        return softcap(scalar_norm(x, w["final.norm"], eps) @ w["head"].T, cfg["logit_softcap"]), after

    def logits(self, tokens):
        return self.run(tokens)[0]
