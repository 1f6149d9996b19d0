"""Plain, slow implementation of the Regesun decoder, the oracle of its tests.

One function per mechanism, whole sequences, no cache, no batching, one token at a time where the
mechanism is a recurrence.  It works on a checkpoint as it is stored (the config.json dictionary and
the tensors by name) in float64 by default, and shares no code with the package under test.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x divided by its root mean square over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def add_normed(x, y, w, scale, eps):
    """The residual with a sublayer's result added: x + scale * (w * y / rms(y))."""
    return x + scale * (rms(y, eps) * w)


def window_attention(q, k, v, scale, window=None, sink=None):
    """q, k [T, H, D], v [T, H, V]: token i attends to itself and the ``window`` - 1 tokens before it
    (None: all of them); ``sink`` [H] joins the denominator without a key or a value."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        lo = 0 if window is None else max(0, i - window + 1)
        for h in range(H):
            s = (k[lo:i + 1, h] @ q[i, h]) * scale
            top = s.max() if sink is None else torch.maximum(s.max(), sink[h])
            e = torch.exp(s - top)
            den = e.sum() if sink is None else e.sum() + torch.exp(sink[h] - top)
            out[i, h] = (e / den) @ v[lo:i + 1, h]
    return out


def causal_conv(x, w, b):
    """x [T, C], w [C, taps] (last column: the current token), b [C]; zeros before the start."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        acc = b.clone()
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                acc = acc + w[:, j] * x[s]
        out[t] = acc
    return out


def ssd_recurrence(x, B, C, dt, A, D, state=None):
    """x [T, H, V], B, C [T, G, N], dt [T, H], A, D [H]: S_t = exp(A dt_t) S_{t-1} + dt_t B_t x_t^T,
    y_t = S_t^T C_t + D x_t, head h on group h // (H / G).  Returns (y, last state [H, N, V])."""
    T, H, V = x.shape
    G, N = B.shape[1:]
    S = torch.zeros(H, N, V, dtype=x.dtype) if state is None else state.clone()
    y = torch.zeros_like(x)
    for t in range(T):
        for h in range(H):
            g = h // (H // G)
            S[h] = torch.exp(A[h] * dt[t, h]) * S[h] + dt[t, h] * torch.outer(B[t, g], x[t, h])
            y[t, h] = C[t, g] @ S[h] + D[h] * x[t, h]
    return y, S


def unit(k):
    return k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)


def delta_decay(z):
    """Decay from its logit: exp(-exp(-1/2) sigmoid(z))."""
    return torch.exp(-math.exp(-0.5) * torch.sigmoid(z))


def delta_recurrence(r, k, v, w, a, state=None):
    """r, k, w, a [T, H, D], v [T, H, V]: S_t = diag(w) S - (a u) (u^T S) + k v^T with S the state before
    the token and u the unit key; o_t = S_t^T r_t.  Returns (o, last state [H, D, V])."""
    T, H, D = k.shape
    S = torch.zeros(H, D, v.shape[2], dtype=k.dtype) if state is None else state.clone()
    out = torch.zeros_like(v)
    for t in range(T):
        for h in range(H):
            u = unit(k[t, h])
            S[h] = w[t, h][:, None] * S[h] - torch.outer(a[t, h] * u, u @ S[h]) + torch.outer(k[t, h], v[t, h])
            out[t, h] = r[t, h] @ S[h]
    return out, S


def clamped_glu(gate, up, limit):
    g, u = torch.clamp(gate, max=limit), torch.clamp(up, -limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def silu(x):
    return x * torch.sigmoid(x)


class Oracle:
    """``cfg``: config.json as a dictionary, ``weights``: name -> tensor."""

    def __init__(self, cfg, weights, dtype=torch.float64):
        self.cfg = cfg
        self.w = {k: v.to(dtype) for k, v in weights.items()}
        self.dtype = dtype
        self.eps = cfg["norm"]["eps"]

    def general_delta(self, p, m, h):
        w, T, H, D = self.w, h.shape[0], m["heads"], m["dim"]
        heads = lambda n: (h @ w[p + n].T).view(T, H, D)  # noqa: E731
        z = torch.tanh(h @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]
        a = torch.sigmoid(h @ w[p + "a"].T + w[p + "a.b"])
        o, _ = delta_recurrence(heads("r"), heads("k"), heads("v"), delta_decay(z).view(T, H, D), a.view(T, H, D))
        o = rms(o, self.eps).reshape(T, H * D) * w[p + "norm"]
        return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T

    def mamba2(self, p, m, h):
        w, T = self.w, h.shape[0]
        H, V, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
        inner = H * V
        proj = h @ w[p + "in"].T
        z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * G * N], proj[:, 2 * inner + 2 * G * N:]
        xbc = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
        dt = torch.nn.functional.softplus(dt + w[p + "dt_bias"], threshold=1e9)
        y, _ = ssd_recurrence(xbc[:, :inner].reshape(T, H, V), xbc[:, inner:inner + G * N].reshape(T, G, N),
                              xbc[:, inner + G * N:].reshape(T, G, N), dt, -torch.exp(w[p + "A_log"]), w[p + "D"])
        y = y.reshape(T, inner) * silu(z)
        y = rms(y.view(T, m["norm_groups"], -1), self.eps).reshape(T, inner) * w[p + "norm"]
        return y @ w[p + "o"].T

    def latent_attention(self, p, m, h):
        w, T, H, D, V = self.w, h.shape[0], m["heads"], m["dim"], m["vdim"]
        q = (h @ w[p + "q"].T).view(T, H, D)
        c = rms(h @ w[p + "dkv"].T, self.eps) * w[p + "dkv.norm"]
        k, v = (c @ w[p + "uk"].T).view(T, H, D), (c @ w[p + "uv"].T).view(T, H, V)
        o = window_attention(q, k, v, m["scale"], m["mask"]["size"], w[p + "sink"]).reshape(T, H * V)
        return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T

    def mlp(self, p, m, h):
        w = self.w
        return clamped_glu(h @ w[p + "gate"].T, h @ w[p + "up"].T, m["limit"]) @ w[p + "down"].T

    def run(self, tokens):
        """(logits [T, vocab], [residual after every layer])."""
        cfg, w, eps = self.cfg, self.w, self.eps
        x = w["embed"][torch.tensor(tokens)] + w["pos"][:len(tokens)]
        after = []
        for i, lay in enumerate(cfg["layers"]):
            p = f"l{i}."
            y = getattr(self, lay["type"])(p + "mix.", lay["mixer"], rms(x, eps) * w[p + "norm1"])
            x = add_normed(x, y, w[p + "norm1b"], w[p + "ls1"], eps)
            if lay.get("mlp"):
                y = self.mlp(p + "mlp.", lay["mlp"], rms(x, eps) * w[p + "norm2"])
                x = add_normed(x, y, w[p + "norm2b"], w[p + "ls2"], eps)
            after.append(x)
        return (rms(x, eps) * w["final.norm"]) @ w["head"].T, after

    def logits(self, tokens):
        return self.run(tokens)[0]
