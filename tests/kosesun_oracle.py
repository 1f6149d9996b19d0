"""Plain, slow implementation of the Kosesun decoder, the oracle of its tests.

One function per mechanism, whole sequences, no cache, no batching, one token at a time where the
mechanism is a recurrence.  It works on a checkpoint as it is stored (the config.json dictionary and
the tensors by name) in float64 by default, and shares no code with the package under test.
"""
from __future__ import annotations

import torch


def rms(x, eps):
    """x divided by its root mean square over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_around_zero(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def hyper_read(streams, w_in):
    """[T, S, W] -> [T, W]: the sublayer's input, a weighted sum of the streams."""
    out = torch.zeros_like(streams[:, 0])
    for s in range(streams.shape[1]):
        out = out + w_in[s] * streams[:, s]
    return out


def hyper_write(streams, y, mix, w_out):
    """New stream t = sum over s of mix[s, t] * stream s, plus w_out[t] * y."""
    new = []
    for t in range(streams.shape[1]):
        x = w_out[t] * y
        for s in range(streams.shape[1]):
            x = x + mix[s, t] * streams[:, s]
        new.append(x)
    return torch.stack(new, 1)


def rotate_interleaved(x, pos, base, dims):
    """x [T, heads, D], pos [T]: dimension 2i turns with dimension 2i + 1."""
    out = x.clone()
    for i in range(dims // 2):
        a = pos.to(x.dtype) * base ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def sink_attention(q, k, v, scale, sink=None):
    """Causal attention, query head h on key / value head h // (H / G); ``sink`` [H] joins the
    softmax's denominator without a key or a value."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype, device=q.device)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        for i in range(T):
            row = s[i, :i + 1]
            top = row.max() if sink is None else torch.maximum(row.max(), sink[h])
            e = torch.exp(row - top)
            den = e.sum() if sink is None else e.sum() + torch.exp(sink[h] - top)
            out[i, h] = (e / den) @ v[:i + 1, g]
    return out


def log_decay(z, tau):
    """log(sigmoid(z) ^ (1 / tau))."""
    return torch.nn.functional.logsigmoid(z) / tau


def gla_recurrence(q, k, v, logd, state=None):
    """q, k, logd [T, H, dk], v [T, H, dv]: o_t = S_t^T q_t with
    S_t = diag(exp(logd_t)) S_{t-1} + k_t v_t^T.  Returns (o, last state [H, dk, dv])."""
    T, H, dk = q.shape
    dv = v.shape[2]
    S = torch.zeros(H, dk, dv, dtype=q.dtype, device=q.device) if state is None else state.clone()
    out = torch.zeros(T, H, dv, dtype=q.dtype, device=q.device)
    for t in range(T):
        S = torch.exp(logd[t])[:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out, S


def relu2(x):
    return torch.clamp(x, min=0) ** 2


def softcap(x, cap):
    return cap * torch.tanh(x / cap)


class Oracle:
    """``cfg``: config.json as a dictionary, ``weights``: name -> tensor."""

    def __init__(self, cfg, weights, dtype=torch.float64):
        self.cfg = cfg
        self.w = {k: v.to(dtype) for k, v in weights.items()}
        self.dtype = dtype

    def attention(self, i, m, h, first):
        w, p, eps = self.w, f"l{i}.mix.", self.cfg["norm"]["eps"]
        T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        q = rms(h @ w[p + "q"].T, eps) * w[p + "q.norm"]
        k = rms(h @ w[p + "k"].T, eps) * w[p + "k.norm"]
        v = h @ w[p + "v"].T
        pos = torch.arange(T)
        q = rotate_interleaved(q.view(T, H, D), pos, m["rot"]["base"], m["rot"]["dims"])
        k = rotate_interleaved(k.view(T, G, D), pos, m["rot"]["base"], m["rot"]["dims"])
        if m.get("v_mix"):
            if first is None:
                first = v
            else:
                lam = w[p + "vmix"]
                v = (1 - lam) * v + lam * first
        o = sink_attention(q, k, v.view(T, G, V), m["scale"], w[p + "sink"])
        o = o * torch.sigmoid(h @ w[p + "g"].T)[:, :, None]
        return o.reshape(T, H * V) @ w[p + "o"].T, first

    def gla(self, i, m, h):
        w, p, eps = self.w, f"l{i}.mix.", self.cfg["norm"]["eps"]
        T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
        q = (h @ w[p + "q"].T).view(T, H, D) * D ** -0.5
        k = (h @ w[p + "k"].T).view(T, H, D)
        v = (h @ w[p + "v"].T).view(T, H, V)
        z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
        o, _ = gla_recurrence(q, k, v, log_decay(z, m["tau"]).view(T, H, D))
        o = (rms(o, eps) * w[p + "norm"]).reshape(T, H * V)
        return (o * torch.nn.functional.silu(h @ w[p + "g"].T)) @ w[p + "o"].T

    def run(self, tokens):
        """(logits [T, vocab], [sum of the streams after every layer])."""
        cfg, w = self.cfg, self.w
        eps = cfg["norm"]["eps"]
        x = w["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
        st = torch.stack([x] * cfg["streams"], 1)
        first, after = None, []
        for i, lay in enumerate(cfg["layers"]):
            p = f"l{i}."
            h = norm_around_zero(hyper_read(st, w[p + "hc1.in"]), w[p + "norm1"], eps)
            if lay["type"] == "attention":
                y, first = self.attention(i, lay["mixer"], h, first)
            else:
                y = self.gla(i, lay["mixer"], h)
            st = hyper_write(st, y, w[p + "hc1.mix"], w[p + "hc1.out"])
            if lay.get("mlp"):
                h = norm_around_zero(hyper_read(st, w[p + "hc2.in"]), w[p + "norm2"], eps)
                y = relu2(h @ w[p + "mlp.up"].T) @ w[p + "mlp.down"].T
                st = hyper_write(st, y, w[p + "hc2.mix"], w[p + "hc2.out"])
            after.append(st.sum(1))
        x = norm_around_zero(st.sum(1), w["final.norm"], eps)
        return softcap(x @ w["head"].T, cfg["logit_softcap"]), after

    def logits(self, tokens):
        return self.run(tokens)[0]
