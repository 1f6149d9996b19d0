"""The mixers' and norms' HIP kernels (mixers.h), one by one, against the plain oracle
(tests/regesun_oracle.py) in fp64 on the same rounded operands, in both element types."""
import numpy as np
import pytest
import torch

import regesun_oracle as orc
from hybrid_util import Step, rel_err
from mlopamd import ops
from mlopamd.runtime.attn_meta import MetaBuffers
from mlopamd.runtime.kv_cache import BLOCK_SIZE, pad_dim

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 2e-5, torch.bfloat16: 1.2e-2}


def rnd(*shape, seed=0, dtype=torch.float32, gain=1.0, mean=0.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * gain + mean).to(dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W", [(1, 64), (5, 330), (3, 75), (300, 1024), (2, 96), (7, 4096), (260, 4104), (270, 8192), (2, 3001)])
def test_residual(gpu, dtype, T, W):
    eps = 1e-4
    table, pos_table = rnd(40, W, seed=1, dtype=dtype), rnd(50, W, seed=2, dtype=dtype)
    ids = torch.randint(0, 40, (T,), generator=torch.Generator().manual_seed(2))
    pos = torch.randint(0, 50, (T,), generator=torch.Generator().manual_seed(4), dtype=torch.int32)
    n1, n2, post = (rnd(W, seed=i, mean=1.0, gain=0.3) for i in (5, 6, 7))
    x, xn = ops.residual_begin(ids.to(gpu), table.to(gpu), 1.7, pos_table.to(gpu), pos.to(gpu), n1.to(gpu), eps)
    ref = 1.7 * table[ids].double() + pos_table[pos.long()].double()
    assert rel_err(x, ref) < 1e-6 and rel_err(xn, orc.rms(ref, eps) * n1.double()) < TOL[dtype]
    for k in range(3):
        y = rnd(T, W, seed=20 + k, dtype=dtype, gain=3.0)
        if k == 2:  # without a norm of its own, and nothing written back
            before = x.clone()
            xn = ops.residual_step(x, y.to(gpu), None, n2.to(gpu), eps, store=False)
            assert torch.equal(before, x)
            ref = ref + y.double()
        else:
            xn = ops.residual_step(x, y.to(gpu), post.to(gpu), n2.to(gpu), eps)
            ref = orc.add_normed(ref, y.double(), post.double(), 1.0, eps)
            assert rel_err(x, ref) < 3e-6
        assert rel_err(xn, orc.rms(ref, eps) * n2.double()) < TOL[dtype]
    x, _ = ops.residual_begin(ids.to(gpu), table.to(gpu), 1.0, None, pos.to(gpu), n1.to(gpu), eps)
    assert torch.equal(x, table[ids].float().to(gpu))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,n,groups,lead", [(3, 192, 4, 0), (70, 96, 1, 3), (5, 1024, 1, 8), (2, 8192, 2, 0), (9, 10240, 1, 16),
                                             (33, 130, 2, 1), (300, 4096, 32, 8), (6, 60, 3, 4), (4, 512, 1, 0), (5, 77, 7, 2)])
def test_gated_norm(gpu, dtype, T, n, groups, lead):
    eps = 1e-3
    y, proj, w = rnd(T, n, seed=1, dtype=dtype), rnd(T, (lead + n + 7) // 8 * 8 + 8, seed=2, dtype=dtype), rnd(n, seed=3, mean=1.0)
    gate = proj.to(gpu)[:, lead:lead + n]
    z = proj[:, lead:lead + n].double()
    norm = lambda v: orc.rms(v.view(T, groups, -1), eps).reshape(T, n) * w.double()  # noqa: E731
    out = ops.gated_norm(y.to(gpu), gate, w.to(gpu), groups, eps, "silu", gate_first=True)
    assert rel_err(out, norm(y.double() * orc.silu(z))) < TOL[dtype]
    out = ops.gated_norm(y.to(gpu), gate, w.to(gpu), groups, eps, "sigmoid", gate_first=False)
    assert rel_err(out, norm(y.double()) * torch.sigmoid(z)) < TOL[dtype]


@pytest.mark.parametrize("M,I,K", [(1, 64, 64), (3, 512, 512), (8, 1024, 1024), (16, 160, 320), (40, 256, 2048), (100, 48, 192),
                                   (300, 192, 320), (700, 1024, 512), (2049, 1152, 384), (4100, 1280, 1024), (33, 32, 72)])
def test_gemm_clamped_unit(gpu, M, I, K):
    """The clamped gated unit in every row regime of the GEMM planner and in fp32, with values on both
    sides of every clamp."""
    x, gate, up = rnd(M, K, seed=1, dtype=torch.bfloat16), *(rnd(I, K, seed=s, dtype=torch.bfloat16, gain=2 * K ** -0.5) for s in (2, 3))
    w = ops.interleave_gate_up(gate, up)
    for alpha, limit in ((1.702, 1.5), (0.9, 4.0)):
        g, u = x.double() @ gate.double().T, x.double() @ up.double().T
        assert limit > 2 or ((g > limit).any() and (u < -limit).any())
        g, u = g.clamp(max=limit), u.clamp(-limit, limit)
        want = g * torch.sigmoid(alpha * g) * (u + 1)
        y = ops.gemm(x.to(gpu), w.to(gpu), epi=ops.EPI_SILU_MUL, glu=(alpha, limit))
        assert rel_err(y, want) < 1.5e-2
        y = ops.gemm(x.float().to(gpu), w.float().to(gpu), epi=ops.EPI_SILU_MUL, glu=(alpha, limit))
        assert rel_err(y, want) < 1e-5
    plain = ops.gemm(x.to(gpu), w.to(gpu), epi=ops.EPI_SILU_MUL)  # the other form is untouched
    g, u = x.double() @ gate.double().T, x.double() @ up.double().T
    assert rel_err(plain, orc.silu(g) * u) < 2e-2


# rows and portions of the recurrent ops: starting and continuing sequences, block and chunk borders
Q_LENS = [1, 1, 2, 3, 15, 16, 17, 64, 65, 150]
CTX = [1, 40, 2, 60, 80, 16, 17, 64, 165, 150]


def _fresh(c, n, state, row):
    return None if c == n else state[row].double()


def _untouched(step, d_state, state):
    for row in set(range(len(state))) - set(step.rows.tolist()):
        assert torch.equal(d_state[row].cpu(), state[row])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C,taps,lead", [(40, 4, 8), (96, 4, 0), (33, 3, 5), (1100, 2, 16), (24, 1, 0), (50, 7, 3), (16, 16, 8)])
def test_short_conv(gpu, dtype, C, taps, lead):
    step = Step(Q_LENS, CTX, gpu)
    proj = rnd(step.T, lead + C + 3 + -(lead + C + 3) % 8, seed=1, dtype=dtype)
    w, b = rnd(C, taps, seed=2), rnd(C, seed=3)
    tail = rnd(len(Q_LENS) + 2, taps - 1, C, seed=4)
    d_tail = tail.to(gpu)
    out = ops.short_conv(proj.to(gpu)[:, lead:lead + C], w.to(gpu), b.to(gpu), d_tail, step.meta)
    for n, c, s, row in zip(step.q_lens, step.ctx, step.starts(), step.rows.tolist()):
        x = proj[s:s + n, lead:lead + C].double()
        old = torch.zeros(taps - 1, C, dtype=torch.float64) if c == n else tail[row].double()
        seq = torch.cat([old, x])
        want = orc.silu(orc.causal_conv(seq, w.double(), b.double())[taps - 1:])
        assert rel_err(out[s:s + n], want) < TOL[dtype], (n, c)
        if taps > 1:
            assert torch.equal(d_tail[row].cpu(), seq[len(seq) - taps + 1:].float()), (n, c)
    _untouched(step, d_tail, tail)


def _ssd_inputs(step, H, V, N, G, dtype, seed=0):
    C = H * V + 2 * G * N
    xbc = rnd(step.T, C, seed=seed + 1, dtype=dtype)
    dt = rnd(step.T, H + -H % 8, seed=seed + 2, dtype=dtype, gain=1.5)
    return xbc, dt, rnd(H, seed=seed + 3, mean=-1.0), -torch.exp(rnd(H, seed=seed + 4, gain=1.5, mean=-1.0)), rnd(H, seed=seed + 5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,V,N,G", [(4, 24, 40, 2), (2, 64, 32, 1), (3, 30, 100, 3), (2, 128, 128, 2), (2, 40, 200, 1),
                                     (1, 17, 300, 1), (6, 16, 16, 2), (1, 129, 5, 1), (16, 48, 64, 4), (40, 128, 24, 8)])
def test_ssd(gpu, dtype, H, V, N, G):
    """Decoded rows and portions in one step, slots that held something else before."""
    step = Step(Q_LENS, CTX, gpu)
    xbc, dt, bias, a_neg, skip = _ssd_inputs(step, H, V, N, G, dtype)
    state = rnd(len(Q_LENS) + 2, H, N, V, seed=9)
    d_state = state.to(gpu)
    y = ops.ssd(xbc.to(gpu), dt.to(gpu)[:, :H], G, bias.to(gpu), a_neg.to(gpu), skip.to(gpu), d_state, step.meta)
    x = xbc.double()
    d = torch.nn.functional.softplus(dt[:, :H].double() + bias.double())
    for n, c, s, row in zip(step.q_lens, step.ctx, step.starts(), step.rows.tolist()):
        v = x[s:s + n]
        want, S = orc.ssd_recurrence(v[:, :H * V].reshape(n, H, V), v[:, H * V:H * V + G * N].reshape(n, G, N),
                                     v[:, H * V + G * N:].reshape(n, G, N), d[s:s + n], a_neg.double(), skip.double(),
                                     _fresh(c, n, state, row))
        assert rel_err(y[s:s + n], want.reshape(n, -1)) < TOL[dtype], (n, c)
        assert rel_err(d_state[row], S) < 3e-5, (n, c)
    _untouched(step, d_state, state)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("bias", [-60.0, 30.0])
def test_ssd_extreme_steps(gpu, dtype, bias):
    """Steps so small that nothing changes, and so large that the state is forgotten at once."""
    H, V, N, G = 2, 20, 24, 1
    step = Step([1, 33], [40, 50], gpu)
    xbc, dt, _, a_neg, skip = _ssd_inputs(step, H, V, N, G, dtype)
    state = rnd(4, H, N, V, seed=9)
    d_state, b = state.to(gpu), torch.full((H,), bias)
    y = ops.ssd(xbc.to(gpu), dt.to(gpu)[:, :H], G, b.to(gpu), a_neg.to(gpu), skip.to(gpu), d_state, step.meta)
    d = torch.nn.functional.softplus(dt[:, :H].double() + b.double())
    for n, s, row in zip(step.q_lens, step.starts(), step.rows.tolist()):
        v = xbc[s:s + n].double()
        want, S = orc.ssd_recurrence(v[:, :H * V].reshape(n, H, V), v[:, H * V:H * V + G * N].reshape(n, G, N),
                                     v[:, H * V + G * N:].reshape(n, G, N), d[s:s + n], a_neg.double(), skip.double(),
                                     state[row].double())
        assert rel_err(y[s:s + n], want.reshape(n, -1)) < TOL[dtype] and rel_err(d_state[row], S) < 3e-5


def _delta_inputs(step, H, dk, dv, rank, dtype, seed=0):
    n = H * (3 * dk + dv) + rank
    proj = rnd(step.T, n + -n % 8 + 8, seed=seed + 1, dtype=dtype)
    w2 = rnd(H * dk, rank, seed=seed + 2, dtype=dtype, gain=2.0 / rank ** 0.5)
    return proj, w2, rnd(H * dk, seed=seed + 3, mean=-1.0, gain=2.0), rnd(H * dk, seed=seed + 4, gain=1.5)


def _delta_oracle(x, H, dk, dv, rank, w2, w0, a_b, scale, state):
    x = x.double()
    T, hk, hv = x.shape[0], H * dk, H * dv
    z = torch.tanh(x[:, 3 * hk + hv:3 * hk + hv + rank]) @ w2.double().T + w0.double()
    w = orc.delta_decay(z) if scale is None else torch.exp(-scale * torch.sigmoid(z))
    a = torch.sigmoid(x[:, 2 * hk + hv:3 * hk + hv] + a_b.double())
    o, S = orc.delta_recurrence(x[:, :hk].reshape(T, H, dk), x[:, hk:2 * hk].reshape(T, H, dk),
                                x[:, 2 * hk:2 * hk + hv].reshape(T, H, dv), w.reshape(T, H, dk), a.reshape(T, H, dk), state)
    return o.reshape(T, hv), S


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dk,dv,rank,scale", [(3, 24, 24, 12, None), (2, 64, 64, 16, None), (1, 100, 100, 5, None),
                                                (2, 128, 128, 64, None), (2, 200, 72, 8, None), (1, 272, 17, 3, None),
                                                (4, 16, 16, 1, 3.0), (2, 8, 129, 20, None), (2, 48, 33, 40, 9.0),
                                                (17, 32, 32, 7, None)])
def test_delta(gpu, dtype, H, dk, dv, rank, scale):
    """Decoded rows and portions in one step, slots that held something else before; other decay
    bounds (past the blocks' range the portions run token by token)."""
    step = Step(Q_LENS, CTX, gpu)
    proj, w2, w0, a_b = _delta_inputs(step, H, dk, dv, rank, dtype)
    state = rnd(len(Q_LENS) + 2, H, dk, dv, seed=9)
    d_state = state.to(gpu)
    o = ops.delta(proj.to(gpu), w2.to(gpu), w0.to(gpu), a_b.to(gpu), scale or float(np.exp(-0.5)), 1e-6, d_state, step.meta)
    for n, c, s, row in zip(step.q_lens, step.ctx, step.starts(), step.rows.tolist()):
        want, S = _delta_oracle(proj[s:s + n], H, dk, dv, rank, w2, w0, a_b, scale, _fresh(c, n, state, row))
        assert rel_err(o[s:s + n], want) < TOL[dtype], (n, c)
        assert rel_err(d_state[row], S) < 3e-5, (n, c)
    _untouched(step, d_state, state)


@pytest.mark.parametrize("dtype", DTYPES)
def test_delta_repeated_keys(gpu, dtype):
    """One key again and again with full removal and no decay: each value replaces the last, and the
    block's triangular system is as far from the identity as it gets."""
    H, dk, dv, rank = 2, 32, 16, 4
    step = Step([70, 1], [70, 30], gpu)
    proj, w2, w0, a_b = _delta_inputs(step, H, dk, dv, rank, dtype)
    proj[:, H * dk:2 * H * dk] = proj[:1, H * dk:2 * H * dk]
    w0, a_b = torch.full_like(w0, -40.0), torch.full_like(a_b, 40.0)
    state = rnd(4, H, dk, dv, seed=9)
    d_state = state.to(gpu)
    o = ops.delta(proj.to(gpu), w2.to(gpu), w0.to(gpu), a_b.to(gpu), float(np.exp(-0.5)), 1e-6, d_state, step.meta)
    for n, c, s, row in zip(step.q_lens, step.ctx, step.starts(), step.rows.tolist()):
        want, S = _delta_oracle(proj[s:s + n], H, dk, dv, rank, w2, w0, a_b, None, _fresh(c, n, state, row))
        assert rel_err(o[s:s + n], want) < TOL[dtype] and rel_err(d_state[row], S) < 3e-5


@pytest.mark.parametrize("dtype", DTYPES)
def test_recurrent_large_step(gpu, dtype):
    """A step with the longer chunks: states that pass through hundreds of blocks, a continued
    sequence, a row beside them."""
    q_lens, ctx = [1, 4000, 99, 130], [30, 4100, 99, 131]
    step = Step(q_lens, ctx, gpu, chunk=64)
    assert step.meta.chunk == 128
    H, V, N, G = 1, 20, 36, 1
    xbc, dt, bias, a_neg, skip = _ssd_inputs(step, H, V, N, G, dtype, seed=40)
    a_neg = a_neg * 0.02  # (memory over hundreds of tokens)
    state = rnd(len(q_lens) + 2, H, N, V, seed=9)
    d_state = state.to(gpu)
    y = ops.ssd(xbc.to(gpu), dt.to(gpu)[:, :H], G, bias.to(gpu), a_neg.to(gpu), skip.to(gpu), d_state, step.meta)
    d = torch.nn.functional.softplus(dt[:, :H].double() + bias.double())
    tail, x = rnd(len(q_lens) + 2, 3, 24, seed=5), rnd(step.T, 24, seed=6, dtype=dtype)
    d_tail, w, b = tail.to(gpu), rnd(24, 4, seed=7), rnd(24, seed=8)
    conv = ops.short_conv(x.to(gpu), w.to(gpu), b.to(gpu), d_tail, step.meta)
    dk, dv, rank = 20, 36, 9
    proj, w2, w0, a_b = _delta_inputs(step, H, dk, dv, rank, dtype, seed=60)
    w0 = w0 - 4
    dst = rnd(len(q_lens) + 2, H, dk, dv, seed=10)
    d_dst = dst.to(gpu)
    o = ops.delta(proj.to(gpu), w2.to(gpu), w0.to(gpu), a_b.to(gpu), float(np.exp(-0.5)), 1e-6, d_dst, step.meta)
    for n, c, s, row in zip(step.q_lens, step.ctx, step.starts(), step.rows.tolist()):
        v = xbc[s:s + n].double()
        want, S = orc.ssd_recurrence(v[:, :H * V].reshape(n, H, V), v[:, H * V:H * V + G * N].reshape(n, G, N),
                                     v[:, H * V + G * N:].reshape(n, G, N), d[s:s + n], a_neg.double(), skip.double(),
                                     _fresh(c, n, state, row))
        assert rel_err(y[s:s + n], want.reshape(n, -1)) < TOL[dtype] and rel_err(d_state[row], S) < 5e-5, (n, c)
        old = torch.zeros(3, 24, dtype=torch.float64) if c == n else tail[row].double()
        want = orc.silu(orc.causal_conv(torch.cat([old, x[s:s + n].double()]), w.double(), b.double())[3:])
        assert rel_err(conv[s:s + n], want) < TOL[dtype]
        want, S = _delta_oracle(proj[s:s + n], H, dk, dv, rank, w2, w0, a_b, None, _fresh(c, n, dst, row))
        assert rel_err(o[s:s + n], want) < TOL[dtype] and rel_err(d_dst[row], S) < 5e-5, (n, c)


def test_graph_padding_rows(gpu):
    """Padding rows of a captured decode step (no context): finite outputs, no state touched."""
    mb = MetaBuffers(8, 8, 4, 16, 2, 64, gpu, flash_min_q=2, flash_tile=128, part_dim=64, chunk=64, expand_window=0)
    mb.bt_h[1, :1] = 1
    mb.fill_decode(np.array([1], np.int32), np.array([1], np.int32), np.zeros(1, np.int64), pad_to=4)
    mb.upload()
    meta = mb.meta(4, 4, 4, 32, 1)
    step = type("S", (), {"T": 4})
    bf = torch.bfloat16

    def check(fn, state):
        d = state.to(gpu)
        out = fn(d)
        assert float(out[1:].abs().max()) == 0 and float(out[0].abs().max()) > 0
        assert torch.equal(d[[0, 2, 3]].cpu(), state[[0, 2, 3]]) and not torch.equal(d[1].cpu(), state[1])

    xbc, dt, bias, a_neg, skip = (t.to(gpu) for t in _ssd_inputs(step, 2, 24, 16, 1, bf))
    check(lambda S: ops.ssd(xbc, dt[:, :2], 1, bias, a_neg, skip, S, meta), rnd(4, 2, 16, 24, seed=9))
    proj, w2, w0, a_b = (t.to(gpu) for t in _delta_inputs(step, 2, 16, 24, 4, bf))
    check(lambda S: ops.delta(proj, w2, w0, a_b, 0.6, 1e-6, S, meta), rnd(4, 2, 16, 24, seed=9))
    x, w, b = rnd(4, 40, seed=1, dtype=bf).to(gpu), rnd(40, 4, seed=2).to(gpu), rnd(40, seed=3).to(gpu)
    check(lambda S: ops.short_conv(x, w, b, S, meta), rnd(4, 3, 40, seed=9))
    cache = torch.zeros(4, 1, BLOCK_SIZE, 64, dtype=bf, device=gpu)
    q, gate = rnd(4, 2, 64, seed=4, dtype=bf).to(gpu), rnd(4, 2 * 24, seed=5, dtype=bf).to(gpu)
    cache[1, 0, 0] = 1.0
    w_kv, w_qk, w_vo = (rnd(*s, seed=i, dtype=bf).to(gpu) for i, s in enumerate([(2 * 128, 64), (2, 64, 64), (2, 24, 64)]))
    out = ops.latent_attention(q, gate, cache, w_kv, w_qk, w_vo, 24, 0.2, 5, None, meta)
    assert float(out[1:].abs().max()) == 0 and float(out[0].abs().max()) > 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("R,lead", [(64, 0), (44, 8), (130, 3), (512, 64), (7, 1)])
def test_latent_store(gpu, dtype, R, lead):
    eps = 1e-3
    step = Step([1, 40, 2], [33, 60, 19], gpu)
    proj, w = rnd(step.T, lead + R + -(lead + R) % 8, seed=1, dtype=dtype), rnd(R, seed=2, mean=1.0)
    cache = torch.zeros(step.num_blocks, 1, BLOCK_SIZE, pad_dim(R), dtype=dtype, device=gpu)
    slots = step.meta.slots.clone()
    slots[0] = -1  # a padding row
    ops.latent_store(proj.to(gpu)[:, lead:lead + R], w.to(gpu), eps, slots, cache)
    s = step.meta.slots.cpu().long()
    got = cache.cpu()[s // BLOCK_SIZE, 0, s % BLOCK_SIZE]
    want = orc.rms(proj[:, lead:lead + R].double(), eps) * w.double()
    assert rel_err(got[1:, :R], want[1:]) < TOL[dtype] and float(got[0].abs().max()) == 0
    assert R == pad_dim(R) or float(cache[..., R:].abs().max()) == 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,H,N,K", [(1, 3, 64, 64), (16, 2, 130, 128), (17, 4, 23, 192), (33, 2, 128, 512), (70, 3, 320, 64),
                                     (150, 2, 28, 128)])
def test_head_mm(gpu, dtype, n, H, N, K):
    """Per-head products of the step's one-token tiles: from tokens to tiles and back, with and without a
    gate, portions beside them."""
    step = Step([1] * n + [5, 2], [7 + i for i in range(n)] + [9, 30], gpu)
    m, T = step.meta, step.T
    x, w, g = rnd(T, H * K + 8, seed=1, dtype=dtype), rnd(H, N, K, seed=2, dtype=dtype, gain=K ** -0.5), rnd(T, H * N + 8, seed=3, dtype=dtype)
    tok = (m.q_start[m.tile_seq.long()] + m.tile_q0).cpu().long()
    want = torch.einsum("thk,hnk->thn", x[:, :H * K].double().view(T, H, K), w.double())
    op, lists = torch.ops.mlop.head_mm, (m.tile_seq, m.tile_q0, m.q_start, m.q_len)
    xd, wd, gd = x.to(gpu)[:, :H * K].unflatten(1, (H, K)), w.to(gpu), g.to(gpu)[:, :H * N]
    out = torch.empty(n, H, N, dtype=dtype, device=gpu)
    op(out, xd, wd, *lists, True, False, None)
    assert rel_err(out, want[tok]) < TOL[dtype]
    back = torch.full((T, H, N), 7.0, dtype=dtype, device=gpu)
    op(back, xd[tok.to(gpu)].contiguous(), wd, *lists, False, True, gd)
    gate = torch.sigmoid(g[:, :H * N].double()).view(T, H, N)
    assert rel_err(back.cpu()[tok], (want * gate)[tok]) < TOL[dtype]
    rest = torch.ones(T, dtype=torch.bool)
    rest[tok] = False
    assert torch.all(back.cpu()[rest] == 7.0)


def _latent_case(gpu, dtype, H, D, V, R, window, q_lens, ctx, min_part=None, spike=False, sink=True, gate=True, seed=0):
    """Max relative error of a latent-attention step against the oracle.  ``spike``: every query asks for
    one key whose score stands out: the first token, the last one inside the window, the first one
    outside it, or the other side of a page border."""
    KP, VP, RP = pad_dim(D), pad_dim(V), pad_dim(R)
    step = Step(q_lens, ctx, gpu, n_kv=-(-H // 16), min_part=min_part, part_dim=RP, seed=seed, expand_window=window)
    scale = 1.7 * D ** -0.5
    uk, uv = rnd(H * D, R, seed=seed + 1, dtype=dtype, gain=R ** -0.5), rnd(H * V, R, seed=seed + 2, dtype=dtype, gain=R ** -0.5)
    w_kv = torch.zeros(H * (KP + VP), RP, dtype=dtype)
    w_qk, w_vo = torch.zeros(H, RP, KP, dtype=dtype), torch.zeros(H, V, RP, dtype=dtype)
    for h in range(H):
        w_kv[h * KP:h * KP + D, :R] = uk[h * D:(h + 1) * D]
        w_kv[H * KP + h * VP:H * KP + h * VP + V, :R] = uv[h * V:(h + 1) * V]
        w_qk[h, :R, :D] = uk[h * D:(h + 1) * D].T
        w_vo[h, :, :R] = uv[h * V:(h + 1) * V]
    cache = torch.zeros(step.num_blocks, 1, BLOCK_SIZE, RP, dtype=dtype)
    q = torch.zeros(step.T, H, KP, dtype=dtype)
    sk = rnd(H, seed=seed + 5, gain=2.0) if sink else None
    gt = rnd(step.T, H * V + 8, seed=seed + 6, dtype=dtype) if gate else None
    want = torch.zeros(step.T, H * V, dtype=torch.float64)
    for i, (n, c, s) in enumerate(zip(step.q_lens, step.ctx, step.starts())):
        lat = rnd(c, 1, R, seed=seed + 10 + i, dtype=dtype)
        k = (lat[:, 0].double() @ uk.double().T).view(c, H, D)
        v = (lat[:, 0].double() @ uv.double().T).view(c, H, V)
        qq = rnd(c, H, D, seed=seed + 50 + i, dtype=dtype)
        if spike:
            for t in range(c - n, c):
                for h in range(H):
                    edge = t - (window or c) + 1
                    j = [0, t, max(0, edge), max(0, edge - 1), max(0, t - t % 16 - 1)][(t + h) % 5]
                    qq[t, h] = (k[j, h] * (14.0 / scale / k[j, h].pow(2).sum())).to(dtype)
        step.scatter(cache, i, lat, c)
        q[s:s + n, :, :D] = qq[c - n:]
        lo = max(0, c - n - window + 1) if window else 0
        o = orc.window_attention(qq[lo:].double(), k[lo:], v[lo:], scale, window or None, sk.double() if sink else None)
        o = o[c - n - lo:].reshape(n, H * V)
        want[s:s + n] = o * torch.sigmoid(gt[s:s + n, :H * V].double()) if gate else o
    out = ops.latent_attention(q.to(gpu), gt.to(gpu)[:, :H * V] if gate else None, cache.to(gpu), w_kv.to(gpu), w_qk.to(gpu),
                               w_vo.to(gpu), V, scale, window, sk.to(gpu) if sink else None, step.meta)
    return max(rel_err(out[s:s + n], want[s:s + n]) for n, s in zip(step.q_lens, step.starts()))


LATENT = [(6, 32, 48, 128), (3, 20, 28, 44), (20, 64, 128, 512), (16, 128, 64, 256), (1, 200, 250, 330), (33, 16, 24, 72),
          (2, 128, 128, 448), (2, 40, 23, 600)]
# bf16: queries and results pass through the latent space rounded once more
LTOL = {torch.float32: 3e-5, torch.bfloat16: 2.5e-2}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,V,R", LATENT)
@pytest.mark.parametrize("window", [0, 1, 23, 64])
def test_latent_attention_mixed_step(gpu, dtype, H, D, V, R, window):
    # decoded tokens and portions down to two tokens, contexts at page, tile and window borders
    q_lens = [1, 1, 1, 1, 1, 1, 2, 3, 31, 130, 17]
    ctx = [1, 16, 17, 24, 65, 161, 2, 67, 31, 150, 48]
    assert _latent_case(gpu, dtype, H, D, V, R, window, q_lens, ctx) < LTOL[dtype]
    assert _latent_case(gpu, dtype, H, D, V, R, window, [1, 5], [40, 21], sink=False, gate=False, seed=3) < LTOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [0, 40, 100])
@pytest.mark.parametrize("H,D,V,R", LATENT[:5])
def test_latent_attention_key_partitions(gpu, dtype, H, D, V, R, window):
    """Split key ranges, also where the op chooses them (long contexts), rows that end before, at and
    behind their borders; twice, so that the tickets re-arm."""
    for _ in range(2):
        assert _latent_case(gpu, dtype, H, D, V, R, window, [1] * 6, [1, 129, 300, 33, 97, 520], min_part=32) < LTOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [0, 1, 16, 33, 50])
@pytest.mark.parametrize("H,D,V,R", [(6, 32, 48, 128), (5, 64, 32, 320)])
def test_latent_attention_one_key_stands_out(gpu, dtype, H, D, V, R, window):
    assert _latent_case(gpu, dtype, H, D, V, R, window, [1, 1, 1, 2, 140, 33], [130, 17, 51, 180, 200, 33], spike=True) < 2 * LTOL[dtype]
    assert _latent_case(gpu, dtype, H, D, V, R, window, [1, 1, 1], [300, 257, 16], spike=True, min_part=64) < 2 * LTOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_attention_long_context(gpu, dtype):
    """Windows of hundreds of tokens over contexts many times as long; far keys stand out."""
    assert _latent_case(gpu, dtype, 2, 64, 48, 96, 600, [1, 500, 1], [1500, 1400, 1025], spike=True) < 2 * LTOL[dtype]
    assert _latent_case(gpu, dtype, 2, 96, 64, 192, 0, [1, 300], [900, 1000]) < LTOL[dtype]
