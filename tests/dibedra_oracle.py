"""Plain, slow implementation of the Dibedra decoder, the oracle of its tests.

One function per mechanism, whole sequences, no cache, no batching.  It works on a checkpoint as it is
stored (the config.json dictionary and the tensors by name) in float64 by default, and shares no code
with the package under test.
"""
from __future__ import annotations

import math

import torch


def dynamic_tanh(x, alpha, w, b):
    """Norm without statistics."""
    return torch.tanh(alpha * x) * w + b


def rms(x, eps):
    """x divided by its root mean square over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def head_norm(x, w, eps):
    """x [T, heads, D]: every head on its own, one weight for all heads."""
    return rms(x, eps) * w


def values_of(k):
    """The values are the projected keys as they are."""
    return k.clone()


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


def window_attention(q, k, v, scale, window):
    """q [T, H, D], k and v [T, G, D]: position i sees itself and the window - 1 positions before it (0: all)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        lo = max(0, i - window + 1) if window else 0
        for h in range(H):
            s = (k[lo:i + 1, h // per] @ q[i, h]) * scale
            e = torch.exp(s - s.max())
            out[i, h] = (e / e.sum()) @ v[lo:i + 1, h // per]
    return out


def output_gate(o, z):
    """One gate per element of the concatenated heads."""
    return o * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def clamped_unit(g, u, limit):
    """The gate is bounded above, the other part on both sides."""
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def softmax_scores(z):
    e = torch.exp(z - z.max())
    return e / e.sum()


def best_groups(choice, count, keep):
    """Indices that the ``keep`` groups with the largest best choice score hold."""
    g = choice.view(count, -1)
    kept = torch.argsort(g.max(-1).values, descending=True)[:keep]
    n = g.shape[1]
    return {int(i) * n + j for i in kept for j in range(n)}


def choose(z, correction, count, keep, top):
    """Router logits of one token -> [(expert, weight)]."""
    s = softmax_scores(z)
    choice = s + correction
    allowed = best_groups(choice, count, keep)
    order = [int(e) for e in torch.argsort(choice, descending=True) if int(e) in allowed]
    return [(e, s[e]) for e in order[:top]]


def identity_expert(h):
    return h


class Oracle:
    """``cfg``: config.json as a dictionary, ``weights``: name -> tensor."""

    def __init__(self, cfg, weights, dtype=torch.float64):
        self.cfg = cfg
        self.w = {k: v.to(dtype) for k, v in weights.items()}
        self.eps = cfg["norm"]["eps"]

    def norm(self, x, name):
        return dynamic_tanh(x, self.w[name + ".alpha"], self.w[name], self.w[name + ".b"])

    def attention(self, p, m, h):
        w, T, H, G, D = self.w, h.shape[0], m["heads"], m["kv_heads"], m["dim"]
        q, k = (h @ w[p + "q"].T).view(T, H, D), (h @ w[p + "k"].T).view(T, G, D)
        v = values_of(k)
        q, k = head_norm(q, w[p + "q.norm"], self.eps), head_norm(k, w[p + "k.norm"], self.eps)
        o = window_attention(rotate(q, m["rot"]), rotate(k, m["rot"]), v, m["scale"], (m.get("mask") or {"size": 0})["size"])
        return output_gate(o.reshape(T, -1), h @ w[p + "g"].T) @ w[p + "o"].T

    def dense(self, p, m, h):
        return gelu_tanh(h @ self.w[p + "up"].T) @ self.w[p + "down"].T

    def expert(self, p, e, limit, h):
        w = self.w
        return clamped_unit(h @ w[f"{p}e{e}.gate"].T, h @ w[f"{p}e{e}.up"].T, limit) @ w[f"{p}e{e}.down"].T

    def moe(self, p, m, h):
        ro, out = m["router"], torch.zeros_like(h)
        z = h @ self.w[p + "router"].T
        groups = ro.get("groups") or {"count": 1, "keep": 1}
        for t in range(h.shape[0]):
            for e, s in choose(z[t], self.w[p + "correction"], groups["count"], groups["keep"], ro["top"]):
                y = self.expert(p, e, m["expert"]["limit"], h[t]) if e < ro["experts"] else identity_expert(h[t])
                out[t] += s * y
        return out

    def run(self, tokens):
        """(logits [T, vocab], [residual after every layer])."""
        cfg = self.cfg
        x = self.w["embed"][torch.tensor(tokens)]
        after = []
        for i, lay in enumerate(cfg["layers"]):
            p = f"l{lay.get('weights_of', i)}."
            h = self.norm(x, p + "norm1")
            y = self.attention(p + "mix.", lay["mixer"], h)
            if lay.get("mlp"):
                y = y + {"dense": self.dense, "moe": self.moe}[lay["mlp"]["kind"]](p + "mlp.", lay["mlp"], h)
            x = x + y
            after.append(x)
        return self.norm(x, "final.norm") @ self.w["head"].T * cfg["logit_scale"], after

    def logits(self, tokens):
        return self.run(tokens)[0]
