"""Plain PyTorch (fp32 math) definitions of every HIP op.

They are the numerics oracle of the GPU tests (``tests/test_kernels_gpu.py``)
and the execution path for CPU tensors, so the scheduler / engine / TP logic is
unit-testable in a GPU-less container.  Layouts match the kernels exactly:
``k_cache[NB, Hkv, BS, D]`` and ``v_cache[NB, Hkv, BS, D]`` (both token-major).
"""
from __future__ import annotations

import math

import torch


def rmsnorm(x, w, eps):
    xf = x.float()
    inv = torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps)
    return (w.float() * (xf * inv).to(x.dtype).float()).to(x.dtype)


def add_rmsnorm(x, residual, w, eps):
    r = (x.float() + residual.float()).to(x.dtype)
    return rmsnorm(r, w, eps), r


def silu_mul(x):
    I = x.shape[-1] // 2
    g, u = x[..., :I].float(), x[..., I:].float()
    return (torch.nn.functional.silu(g).to(x.dtype).float() * u).to(x.dtype)


def embedding(ids, table, vocab_start=0):
    ids = ids.reshape(-1).long()
    local = ids - vocab_start
    ok = (local >= 0) & (local < table.shape[0])
    out = table[local.clamp(0, table.shape[0] - 1)].clone()
    out[~ok] = 0
    return out


def rotate(x, cos, sin):
    half = x.shape[-1] // 2
    x1, x2 = x[..., :half], x[..., half:]
    return torch.cat([x1 * cos - x2 * sin, x2 * cos + x1 * sin], dim=-1)


def rope_cache(qkv, positions, cos_sin, slots, k_cache, v_cache, n_q_heads):
    """Rotate q/k, scatter k/v into the paged cache, return q [T, Hq, D]."""
    T = qkv.shape[0]
    Hkv, BS, D = k_cache.shape[1], k_cache.shape[2], k_cache.shape[3]
    half = D // 2
    x = qkv[:, : (n_q_heads + 2 * Hkv) * D].float().view(T, n_q_heads + 2 * Hkv, D)
    cs = cos_sin[positions.long()].float()  # [T, D]
    cos, sin = cs[:, None, :half], cs[:, None, half:]
    q = rotate(x[:, :n_q_heads], cos, sin).to(qkv.dtype)
    k = rotate(x[:, n_q_heads:n_q_heads + Hkv], cos, sin).to(qkv.dtype)
    v = x[:, n_q_heads + Hkv:].to(qkv.dtype)
    for t in range(T):
        s = int(slots[t])
        if s < 0:
            continue
        b, o = divmod(s, BS)
        k_cache[b, :, o, :] = k[t]
        v_cache[b, :, o, :] = v[t]
    return q


def gather_kv(k_cache, v_cache, block_table, n):
    """Contiguous K, V [n, Hkv, D] of one sequence from its pages."""
    BS = k_cache.shape[2]
    pages = [int(p) for p in block_table[: (n + BS - 1) // BS]]
    if not pages:
        Hkv, D = k_cache.shape[1], k_cache.shape[3]
        z = torch.zeros(0, Hkv, D, dtype=k_cache.dtype, device=k_cache.device)
        return z, z
    k = torch.cat([k_cache[p].permute(1, 0, 2) for p in pages], 0)[:n]          # [n, Hkv, D]
    v = torch.cat([v_cache[p].permute(1, 0, 2) for p in pages], 0)[:n]          # [n, Hkv, D]
    return k, v


def paged_attention(q, k_cache, v_cache, meta):
    """Causal GQA attention of every query token of ``meta`` over its paged context."""
    out = torch.zeros_like(q)
    Hq, D = q.shape[1], q.shape[2]
    Hkv = k_cache.shape[1]
    G = Hq // Hkv
    scale = 1.0 / math.sqrt(D)
    qs, ql, cl = (meta.q_start.cpu().tolist(), meta.q_len.cpu().tolist(), meta.ctx_len.cpu().tolist())
    bt = meta.block_tables.cpu()
    # only rows referenced by this launch's tiles are live (other rows hold stale values)
    live = set(meta.tile_seq.cpu().tolist())
    if getattr(meta, "ptile_seq", None) is not None:
        live |= set(meta.ptile_seq.cpu().tolist())
    for s in sorted(live):
        if ql[s] == 0 or cl[s] == 0:
            continue
        k, v = gather_kv(k_cache, v_cache, bt[s], cl[s])
        k = k.float().repeat_interleave(G, dim=1)  # [n, Hq, D]
        v = v.float().repeat_interleave(G, dim=1)
        qq = q[qs[s]:qs[s] + ql[s]].float()      # [ql, Hq, D]
        scores = torch.einsum("qhd,khd->hqk", qq, k) * scale
        pos = torch.arange(cl[s] - ql[s], cl[s], device=q.device)[:, None]
        keys = torch.arange(cl[s], device=q.device)[None, :]
        scores = scores.masked_fill((keys > pos)[None], float("-inf"))
        p = torch.softmax(scores, dim=-1)
        out[qs[s]:qs[s] + ql[s]] = torch.einsum("hqk,khd->qhd", p, v).to(q.dtype)
    return out


# ------------------------------------------------- hybrid decoder layers --

def _unit(x, eps):
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def hyper_begin(ids, table, scale, n_streams, w_in, norm_w, eps):
    x = table[ids.reshape(-1).long()].float() * scale
    streams = x[:, None, :].repeat(1, n_streams, 1)
    return streams, (_unit(torch.einsum("s,tsw->tw", w_in, streams), eps) * norm_w).to(table.dtype)


def hyper_step(streams, y, mix, w_out, w_in, norm_w, eps):
    streams.copy_(torch.einsum("st,bsw->btw", mix, streams) + w_out[None, :, None] * y.float()[:, None, :])
    return (_unit(torch.einsum("s,tsw->tw", w_in, streams), eps) * norm_w).to(y.dtype)


def relu2(x):
    return torch.relu(x.float()).square().to(x.dtype)


def xielu(x, a, b):
    z = x.float()
    return (torch.where(z > 0, a * z * z, b * (torch.expm1(z.clamp(max=0)) - z)) + 0.5 * z).to(x.dtype)


def gelu_tanh(x):
    v = x.float()
    return (0.5 * v * (1 + torch.tanh(math.sqrt(2 / math.pi) * (v + 0.044715 * v ** 3)))).to(x.dtype)


def softcap(x, cap):
    return cap * torch.tanh(x.float() / cap)


def rotate_pairs(x, cos, sin):
    """x [T, heads, D] with pairs (2i, 2i + 1), cos / sin [T, R / 2]: the first R dims turn."""
    R = 2 * cos.shape[-1]
    u, v = x[..., :R:2], x[..., 1:R:2]
    c, s = cos[:, None], sin[:, None]
    turned = torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2)
    return torch.cat([turned, x[..., R:]], -1)


def qk_norm_rope(proj, H, D, V, q_w, k_w, eps, cos_sin, positions, slots, k_cache, v_cache, v_first, lam):
    T, G, BS, KP = proj.shape[0], k_cache.shape[1], k_cache.shape[2], k_cache.shape[3]
    x = proj.float()
    q, k, v = x[:, :H * D], x[:, H * D:(H + G) * D], x[:, (H + G) * D:(H + G) * D + G * V]
    if q_w is not None:
        q, k = _unit(q, eps) * q_w, _unit(k, eps) * k_w
    half = cos_sin.shape[1] // 2
    cs = cos_sin[positions.long()]
    q = rotate_pairs(q.reshape(T, H, D), cs[:, :half], cs[:, half:])
    k = rotate_pairs(k.reshape(T, G, D), cs[:, :half], cs[:, half:])
    if v_first is not None:
        v = (1 - lam) * v + lam * v_first.float()
    keep = slots >= 0
    blk, off = slots[keep].long() // BS, slots[keep].long() % BS
    k_cache[blk, :, off, :D] = k[keep].to(k_cache.dtype)
    v_cache[blk, :, off, :V] = v.reshape(T, G, V)[keep].to(v_cache.dtype)
    out = torch.zeros(T, H, KP, dtype=proj.dtype, device=proj.device)
    out[:, :, :D] = q.to(proj.dtype)
    return out


def _live_rows(meta):
    rows = set(meta.tile_seq.tolist()) | set(meta.ptile_seq.tolist())
    qs, ql, cl = meta.q_start.tolist(), meta.q_len.tolist(), meta.ctx_len.tolist()
    return [(r, qs[r], ql[r], cl[r]) for r in sorted(rows) if ql[r] and cl[r]]


def qk_head_norm(q, k, v, H, D, V, q_w, k_w, eps, cos_sin, positions, slots, k_cache, v_cache):
    T, G, half = q.shape[0], k_cache.shape[1], cos_sin.shape[1] // 2
    cs = cos_sin[positions.long()]
    turn = lambda x, n, w: rotate_pairs(_unit(x.float().reshape(T, n, D), eps) * w, cs[:, :half], cs[:, half:]).to(q.dtype)  # noqa: E731
    out = torch.zeros(T, H, k_cache.shape[3], dtype=q.dtype, device=q.device)
    out[:, :, :D] = turn(q, H, q_w)
    keep, BS = slots >= 0, k_cache.shape[2]
    s = slots[keep].long()
    k_cache[s // BS, :, s % BS, :D] = turn(k, G, k_w)[keep]
    v_cache[s // BS, :, s % BS, :V] = (k if v is None else v).reshape(T, G, V)[keep].to(v_cache.dtype)
    return out


def attention_hd(q, k_cache, v_cache, meta, D, V, scale, sink, gate, window=0):
    T, H = q.shape[:2]
    G = k_cache.shape[1]
    out = torch.zeros(T, H, V, dtype=torch.float32, device=q.device)
    for row, s, n, ctx in _live_rows(meta):
        k, v = gather_kv(k_cache, v_cache, meta.block_tables[row], ctx)
        k = k[..., :D].float().repeat_interleave(H // G, 1)
        v = v[..., :V].float().repeat_interleave(H // G, 1)
        w = torch.einsum("qhd,khd->hqk", q[s:s + n, :, :D].float(), k) * scale
        pos = torch.arange(ctx - n, ctx, device=q.device)[:, None]
        keys = torch.arange(ctx, device=q.device)[None]
        hidden = (keys > pos) | (keys <= pos - window) if window else keys > pos
        w = w.masked_fill(hidden[None], float("-inf"))
        if sink is not None:
            w = torch.cat([w, sink.float().view(H, 1, 1).expand(H, n, 1)], -1)
        p = torch.softmax(w, -1)[..., :ctx]
        out[s:s + n] = torch.einsum("hqk,khd->qhd", p, v)
    if gate is not None:
        out = out * torch.sigmoid(gate.float()).view(T, H, -1)
    return out.to(q.dtype)


def gla(proj, H, D, V, a2, a2_b, norm_w, tau, eps, state, meta):
    T, hk, hv = proj.shape[0], H * D, H * V
    x = proj.float()
    q = x[:, :hk].reshape(T, H, D) * D ** -0.5
    k = x[:, hk:2 * hk].reshape(T, H, D)
    v = x[:, 2 * hk:2 * hk + hv].reshape(T, H, V)
    g = x[:, 2 * hk + hv:2 * hk + 2 * hv]
    z = x[:, 2 * hk + 2 * hv:2 * hk + 2 * hv + a2.shape[1]] @ a2.float().t() + a2_b
    decay = torch.exp(torch.nn.functional.logsigmoid(z) / tau).reshape(T, H, D)
    o = torch.zeros(T, H, V, dtype=torch.float32, device=proj.device)
    for row, s, n, ctx in _live_rows(meta):
        S = torch.zeros_like(state[row]) if ctx == n else state[row]
        for t in range(s, s + n):
            S = decay[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
            o[t] = torch.einsum("hdv,hd->hv", S, q[t])
        state[row] = S
    o = (_unit(o, eps) * norm_w).reshape(T, hv) * torch.nn.functional.silu(g)
    return o.to(proj.dtype)


def _unit_n(x, eps, width):
    """x over the root mean square of its first ``width`` columns (the rest are zero)."""
    return x * torch.rsqrt(x.pow(2).sum(-1, keepdim=True) / (width or x.shape[-1]) + eps)


def _next_input(x, norm_w, eps, width, tanh):
    if tanh is not None:
        return norm_w * torch.tanh(tanh[0] * x) + tanh[1]
    return x if norm_w is None else _unit_n(x, eps, width) * norm_w


def residual_begin(ids, table, scale, pos_table, positions, norm_w, eps, width=None, tanh=None):
    x = table[ids.reshape(-1).long()].float() * scale
    if pos_table is not None:
        x = x + pos_table[positions.long()].float()
    return x, _next_input(x, norm_w, eps, width, tanh).to(table.dtype)


def residual_step(x, y, post_w, norm_w, eps, width=None, experts=None, share=None, tanh=None):
    dtype = y.dtype if experts is None else experts[0].dtype
    out = y.float() if y is not None else torch.zeros_like(x)
    if experts is not None:
        rows, inv, gate = experts
        if gate is not None:
            out = out * gate[:, None]
        w = (inv >= 0).float() if share is None else share[0] * (inv >= 0)
        out = out + (rows.float()[inv.long().clamp(min=0)] * w[..., None]).sum(1)
        if share is not None and share[1] is not None:
            out = out + share[2][:, None] * share[1].float()
    x.add_(_unit_n(out, eps, width) * post_w if post_w is not None else out)
    return _next_input(x, norm_w, eps, width, tanh).to(dtype)


def gated_norm(y, gate, w, groups, eps, silu, gate_first):
    T, n = y.shape
    v, g = y.float(), gate.float()
    g = torch.nn.functional.silu(g) if silu else torch.sigmoid(g)
    if gate_first:
        v = v * g
    v = _unit(v.reshape(T, groups, -1), eps).reshape(T, n) * w
    return (v if gate_first else v * g).to(y.dtype)


def clamp_glu(x, alpha, limit):
    """x [T, 2 I] = [gate | up]."""
    g, u = x.float().chunk(2, -1)
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return (g * torch.sigmoid(alpha * g) * (u + 1)).to(x.dtype)


def short_conv(x, w, b, tail, meta):
    out = torch.zeros(x.shape, dtype=torch.float32, device=x.device)
    P = w.shape[1] - 1
    for row, s, n, ctx in _live_rows(meta):
        old = torch.zeros_like(tail[row]) if ctx == n else tail[row]
        seq = torch.cat([old, x[s:s + n].float()], 0)
        for j in range(P + 1):
            out[s:s + n] += seq[j:j + n] * w[:, j]
        tail[row] = seq[len(seq) - P:]
    if b is not None:
        out = out + b
    return torch.nn.functional.silu(out).to(x.dtype)


def ssd(xbc, dt, G, dt_bias, a_neg, d_skip, state, meta):
    _, H, N, V = state.shape
    T = xbc.shape[0]
    v = xbc.float()
    x = v[:, :H * V].reshape(T, H, V)
    B = v[:, H * V:H * V + G * N].reshape(T, G, N).repeat_interleave(H // G, 1)
    C = v[:, H * V + G * N:].reshape(T, G, N).repeat_interleave(H // G, 1)
    d = torch.nn.functional.softplus(dt.float() + dt_bias, threshold=1e9)
    y = torch.zeros(T, H, V, dtype=torch.float32, device=xbc.device)
    for row, s, n, ctx in _live_rows(meta):
        S = torch.zeros_like(state[row]) if ctx == n else state[row]
        for t in range(s, s + n):
            S = torch.exp(a_neg * d[t])[:, None, None] * S + (d[t][:, None] * B[t])[:, :, None] * x[t][:, None, :]
            y[t] = torch.einsum("hnv,hn->hv", S, C[t]) + d_skip[:, None] * x[t]
        state[row] = S
    return y.reshape(T, H * V).to(xbc.dtype)


def delta(proj, w2, w0, a_b, decay_scale, unit_eps, state, meta):
    _, H, D, V = state.shape
    T, hk, hv = proj.shape[0], H * D, H * V
    x = proj.float()
    r, k = x[:, :hk].reshape(T, H, D), x[:, hk:2 * hk].reshape(T, H, D)
    v = x[:, 2 * hk:2 * hk + hv].reshape(T, H, V)
    a = torch.sigmoid(x[:, 2 * hk + hv:3 * hk + hv] + a_b).reshape(T, H, D)
    z = torch.tanh(x[:, 3 * hk + hv:3 * hk + hv + w2.shape[1]]) @ w2.float().t() + w0
    w = torch.exp(-decay_scale * torch.sigmoid(z)).reshape(T, H, D)
    u = k * torch.rsqrt(k.pow(2).sum(-1, keepdim=True) + unit_eps)
    o = torch.zeros(T, H, V, dtype=torch.float32, device=proj.device)
    for row, s, n, ctx in _live_rows(meta):
        S = torch.zeros_like(state[row]) if ctx == n else state[row]
        for t in range(s, s + n):
            z_t = torch.einsum("hd,hdv->hv", u[t], S)
            S = w[t][:, :, None] * S - (a[t] * u[t])[:, :, None] * z_t[:, None, :] + k[t][:, :, None] * v[t][:, None, :]
            o[t] = torch.einsum("hdv,hd->hv", S, r[t])
        state[row] = S
    return o.reshape(T, hv).to(proj.dtype)


def latent_query(x, w, eps, size):
    return torch.nn.functional.pad(_unit(x.float(), eps) * w, (0, size - x.shape[1])).to(x.dtype)


def latent_store(latents, w, eps, slots, cache, rope=None, query=None):
    c = (_unit(latents.float(), eps) * w).to(cache.dtype)
    keep = slots >= 0
    rows = cache.view(-1, cache.shape[-1])
    rows[slots[keep].long(), :c.shape[1]] = c[keep]
    if rope is not None:
        k, table, positions, off = rope
        cs, half = table[positions.long()], table.shape[1] // 2
        k = rotate_pairs(k.float()[:, None], cs[:, :half], cs[:, half:])[:, 0].to(cache.dtype)
        rows[slots[keep].long(), off:off + k.shape[1]] = k[keep]
    return latent_query(*query[:2], eps, query[2]) if query is not None else None


def latent_attention(q, gate, cache, w_kv, H, V, scale, window, sink, meta, rope=None):
    """q [T, H, KP]; w_kv [H (KP + VP), RP]: a head's keys, then values, of a latent row."""
    T, KP = q.shape[0], q.shape[2]
    VP = w_kv.shape[0] // H - KP
    if rope is not None:
        table, n, off, _ = rope
        cs = table[meta.positions.long()]
        turned = rotate_pairs(q[:, :, off:off + n].float(), cs[:, :n // 2], cs[:, n // 2:]).to(q.dtype)
        q = torch.cat([q[:, :, :off], turned, q[:, :, off + n:]], 2)
    out = torch.zeros(T, H, V, dtype=torch.float32, device=q.device)
    for row, s, n, ctx in _live_rows(meta):
        c, _ = gather_kv(cache, cache, meta.block_tables[row], ctx)
        kv = c[:, 0].float() @ w_kv.float().t()
        k = kv[:, :H * KP].reshape(ctx, H, KP)
        v = kv[:, H * KP:].reshape(ctx, H, VP)[..., :V]
        sc = torch.einsum("qhd,khd->hqk", q[s:s + n].float(), k) * scale
        pos = torch.arange(ctx - n, ctx, device=q.device)[:, None]
        keys = torch.arange(ctx, device=q.device)[None]
        hidden = keys > pos
        if window:
            hidden = hidden | (keys <= pos - window)
        sc = sc.masked_fill(hidden[None], float("-inf"))
        if sink is not None:
            sc = torch.cat([sc, sink.float().view(H, 1, 1).expand(H, n, 1)], -1)
        out[s:s + n] = torch.einsum("hqk,khd->qhd", torch.softmax(sc, -1)[..., :ctx], v)
    out = out.reshape(T, H * V)
    if gate is not None:
        out = out * torch.sigmoid(gate.float())
    return out.to(q.dtype)


# ------------------------------------------------------------------ MoE --

def moe_route(logits, top_k):
    p = torch.softmax(logits.float(), dim=-1)
    w, idx = torch.topk(p, top_k, dim=-1)
    w = w / w.sum(-1, keepdim=True)
    return w, idx.to(torch.int32)


def moe_route_sigmoid(logits, E, top_k):
    """fp32 logits [T, E] or, with a gate behind them, [T, E + 1] -> (scores of the top_k largest, experts,
    sigmoid of the gate or None)."""
    s = torch.sigmoid(logits.float())
    w, idx = torch.topk(s[:, :E], top_k, dim=-1)
    return w, idx.to(torch.int32), s[:, E].contiguous() if s.shape[1] > E else None


def moe_route_groups(logits, correction, E, top_k, groups, keep):
    """fp32 logits [T, n] -> (weights, experts [T, k], weight of the outputs past the E experts per token or None)."""
    T, n = logits.shape
    s = torch.softmax(logits.float(), -1)
    choice = s if correction is None else s + correction
    best = choice.view(T, groups, -1).amax(-1)
    kept = torch.zeros_like(best, dtype=torch.bool).scatter_(1, torch.topk(best, keep, -1).indices, True)
    choice = choice.masked_fill(~kept.repeat_interleave(n // groups, 1), float("-inf"))
    idx = torch.topk(choice, top_k, -1).indices
    w = s.gather(1, idx)
    return w, idx.to(torch.int32), (w * (idx >= E)).sum(-1) if n > E else None


def moe_permute(x, topi, e0, n_local):
    """Rows routed to local experts, grouped by expert (stable in slot order), padded to T*k rows.
    Returns (xp [T*k, H], offsets int32 [n_local+1], src int32 [T*k], inv int32 [T*k])."""
    T, k = topi.shape
    flat = topi.reshape(-1).long() - e0
    ok = (flat >= 0) & (flat < n_local)
    slots = torch.nonzero(ok, as_tuple=True)[0]
    e = flat[slots]
    order = torch.argsort(e, stable=True)
    slots, e = slots[order], e[order]
    n = slots.numel()
    counts = torch.bincount(e, minlength=n_local)
    offsets = torch.zeros(n_local + 1, dtype=torch.int32, device=x.device)
    offsets[1:] = torch.cumsum(counts, 0).to(torch.int32)
    xp = torch.zeros(T * k, x.shape[1], dtype=x.dtype, device=x.device)
    xp[:n] = x[slots // k]
    src = torch.full((T * k,), -1, dtype=torch.int32, device=x.device)
    src[:n] = slots.to(torch.int32)
    inv = torch.full((T * k,), -1, dtype=torch.int32, device=x.device)
    inv[slots] = torch.arange(n, dtype=torch.int32, device=x.device)
    return xp, offsets, src, inv


def grouped_gemm(xp, w, offsets):
    """Per group e: rows [off[e], off[e+1]) of xp times w[e]^T (w: [E, N, K]); other rows 0."""
    out = torch.zeros(xp.shape[0], w.shape[1], dtype=xp.dtype, device=xp.device)
    off = offsets.tolist()
    for e in range(w.shape[0]):
        a, b = off[e], off[e + 1]
        if b > a:
            out[a:b] = (xp[a:b].float() @ w[e].float().t()).to(xp.dtype)
    return out


def moe_combine(y, inv, topw):
    T, k = topw.shape
    out = torch.zeros(T, y.shape[1], dtype=torch.float32, device=y.device)
    inv = inv.long().view(T, k)
    for j in range(k):
        ok = inv[:, j] >= 0
        if ok.any():
            out[ok] += topw[ok, j, None].float() * y[inv[ok, j]].float()
    return out.to(y.dtype)
