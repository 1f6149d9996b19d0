"""The hybrid decoder's HIP kernels, one by one, against the plain oracle (tests/kosesun_oracle.py) in
fp64 on the same rounded operands, in both element types."""
import numpy as np
import pytest
import torch

import kosesun_oracle as orc
from hybrid_util import Step, rel_err
from mlopamd import ops
from mlopamd.models.layers import rope_table
from mlopamd.runtime.kv_cache import BLOCK_SIZE, pad_dim

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 2e-5, torch.bfloat16: 1.2e-2}


def rnd(*shape, seed=0, dtype=torch.float32, gain=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * gain).to(dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,S,W", [(1, 1, 64), (5, 2, 330), (3, 3, 75), (300, 4, 1024), (2, 5, 96), (7, 6, 132),
                                   (4, 8, 4096), (2, 11, 50)])
def test_hyper_connections(gpu, dtype, T, S, W):
    eps = 1e-4
    table, ids = rnd(40, W, seed=1, dtype=dtype), torch.randint(0, 40, (T,), generator=torch.Generator().manual_seed(2))
    w = {k: rnd(*sh, seed=i + 3) for i, (k, sh) in enumerate({"in1": (S,), "in2": (S,), "out": (S,), "mix": (S, S),
                                                              "n1": (W,), "n2": (W,)}.items())}
    d = {k: v.to(gpu) for k, v in w.items()}
    f = {k: v.double() for k, v in w.items()}
    st, xn = ops.hyper_begin(ids.to(gpu), table.to(gpu), 2.5, S, d["in1"], d["n1"], eps)
    ref = torch.stack([table[ids].double() * 2.5] * S, 1)
    assert rel_err(st, ref) < 1e-6
    assert rel_err(xn, orc.rms(orc.hyper_read(ref, f["in1"]), eps) * f["n1"]) < TOL[dtype]
    for k in range(2):  # the second time the streams differ from one another
        y = rnd(T, W, seed=20 + k, dtype=dtype)
        xn = ops.hyper_step(st, y.to(gpu), d["mix"], d["out"], d["in2"], d["n2"], eps)
        ref = orc.hyper_write(ref, y.double(), f["mix"], f["out"])
        assert rel_err(st, ref) < 3e-6
        assert rel_err(xn, orc.rms(orc.hyper_read(ref, f["in2"]), eps) * f["n2"]) < TOL[dtype]
    before = st.clone()
    xn = ops.hyper_step(st, y.to(gpu), d["mix"], d["out"], d["in2"], d["n2"], eps, store=False)
    assert torch.equal(before, st)
    ref = orc.hyper_write(ref, y.double(), f["mix"], f["out"])
    assert rel_err(xn, orc.rms(orc.hyper_read(ref, f["in2"]), eps) * f["n2"]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [8, 77, 4096])
def test_relu2_softcap(gpu, dtype, n):
    x = rnd(n, seed=1, dtype=dtype, gain=3.0)
    assert rel_err(ops.softcap(x.to(gpu), 2.5), orc.softcap(x.double(), 2.5)) < 1e-5
    assert rel_err(ops.relu2(x.to(gpu)), orc.relu2(x.double())) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,V,R", [(6, 2, 32, 48, 32), (8, 2, 96, 40, 64), (5, 5, 22, 7, 10), (4, 1, 128, 256, 0),
                                       (3, 1, 72, 64, 72)])
def test_qk_norm_rope(gpu, dtype, H, G, D, V, R):
    eps, base = 1e-3, 5000.0
    step = Step([1, 40, 2], [33, 60, 19], gpu)
    T, nq, nk, nv = step.T, H * D, G * D, G * V
    N = (nq + nk + nv + 9 + 7) // 8 * 8
    proj, vf = rnd(T, N, seed=1, dtype=dtype), rnd(T, nv, seed=2, dtype=dtype)
    qw, kw = 1 + rnd(nq, seed=3, gain=0.3), 1 + rnd(nk, seed=4, gain=0.3)
    lam = torch.tensor([0.35])
    pos = step.meta.positions.cpu().long()
    x = proj.double()
    for norm, mix in ((True, True), (False, False)):
        kc = torch.zeros(step.num_blocks, G, BLOCK_SIZE, pad_dim(D), dtype=dtype, device=gpu)
        vc = torch.zeros(step.num_blocks, G, BLOCK_SIZE, pad_dim(V), dtype=dtype, device=gpu)
        q = ops.qk_norm_rope(proj.to(gpu), H, D, V, qw.to(gpu) if norm else None, kw.to(gpu) if norm else None, eps,
                             rope_table(R, 64, base, device=gpu), step.meta.positions, step.meta.slots, kc, vc,
                             v_first=vf.to(gpu) if mix else None, lam=lam.to(gpu) if mix else None)
        qr, kr, vr = x[:, :nq], x[:, nq:nq + nk], x[:, nq + nk:nq + nk + nv]
        if norm:
            qr, kr = orc.rms(qr, eps) * qw.double(), orc.rms(kr, eps) * kw.double()
        if mix:
            vr = (1 - float(lam)) * vr + float(lam) * vf.double()
        qr = orc.rotate_interleaved(qr.reshape(T, H, D), pos, base, R)
        kr = orc.rotate_interleaved(kr.reshape(T, G, D), pos, base, R)
        assert rel_err(q[:, :, :D], qr) < TOL[dtype]
        assert pad_dim(D) == D or float(q[:, :, D:].abs().max()) == 0
        slots = step.meta.slots.cpu().long()
        got_k = kc.cpu()[slots // BLOCK_SIZE, :, slots % BLOCK_SIZE]
        got_v = vc.cpu()[slots // BLOCK_SIZE, :, slots % BLOCK_SIZE]
        assert rel_err(got_k[..., :D], kr) < TOL[dtype]
        assert rel_err(got_v[..., :V], vr.reshape(T, G, V)) < TOL[dtype]


def _attention_case(gpu, dtype, H, G, D, V, q_lens, ctx, sink=True, gate=True, min_part=None, spike=False, seed=0):
    """Max relative error of a step against the oracle.  ``spike``: every query asks for one far key
    whose score stands out (the first token, or the other side of a page border)."""
    units = G * -(-(H // G) // 16)
    step = Step(q_lens, ctx, gpu, n_kv=units, min_part=min_part, part_dim=pad_dim(V), seed=seed)
    scale = 1.7 * D ** -0.5
    kc = torch.zeros(step.num_blocks, G, BLOCK_SIZE, pad_dim(D), dtype=dtype)
    vc = torch.zeros(step.num_blocks, G, BLOCK_SIZE, pad_dim(V), dtype=dtype)
    q = torch.zeros(step.T, H, pad_dim(D), dtype=dtype)
    sk = rnd(H, seed=seed + 5, gain=2.0) if sink else None
    gt = rnd(step.T, H + 3, seed=seed + 6, dtype=dtype) if gate else None
    want = torch.zeros(step.T, H, V, dtype=torch.float64)
    for i, (n, c, s) in enumerate(zip(step.q_lens, step.ctx, step.starts())):
        k, v = rnd(c, G, D, seed=seed + 10 + i, dtype=dtype), rnd(c, G, V, seed=seed + 30 + i, dtype=dtype)
        qq = rnd(c, H, D, seed=seed + 50 + i, dtype=dtype)
        if spike:  # query t's head h points at one key: its score beats all others together
            for t in range(c - n, c):
                for h in range(H):
                    j = [0, t, max(0, t - t % 16 - 1), t // 2][(t + h) % 4]
                    kj = k[j, h // (H // G)].float()
                    qq[t, h] = (kj * (14.0 / scale / kj.pow(2).sum())).to(dtype)
        step.scatter(kc, i, k, c)
        step.scatter(vc, i, v, c)
        q[s:s + n, :, :D] = qq[c - n:]
        o = orc.sink_attention(qq.double(), k.double(), v.double(), scale, sk.double() if sink else None)[c - n:]
        if gate:
            o = o * torch.sigmoid(gt[s:s + n, :H].double())[..., None]
        want[s:s + n] = o
    out = ops.attention_hd(q.to(gpu), kc.to(gpu), vc.to(gpu), step.meta, D, V, scale,
                           sink=sk.to(gpu) if sink else None, gate=gt.to(gpu)[:, :H] if gate else None)
    return max(rel_err(out[s:s + n], want[s:s + n]) for n, s in zip(step.q_lens, step.starts()))


SIZES = [(6, 2, 32, 48), (8, 2, 96, 40), (20, 1, 64, 128), (5, 5, 128, 64), (4, 1, 192, 256), (3, 1, 256, 192),
         (7, 7, 40, 23), (4, 2, 128, 128), (2, 1, 320, 40), (2, 2, 30, 300)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,V", SIZES)
def test_attention_hd_mixed_step(gpu, dtype, H, G, D, V):
    # decoded tokens and portions down to two tokens, contexts at page and tile borders
    q_lens = [1, 1, 1, 1, 1, 2, 3, 31, 130, 17]
    ctx = [1, 16, 17, 32, 161, 2, 67, 31, 150, 48]
    assert _attention_case(gpu, dtype, H, G, D, V, q_lens, ctx) < TOL[dtype]
    assert _attention_case(gpu, dtype, H, G, D, V, [1, 5], [40, 21], sink=False, gate=False, seed=3) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,V", SIZES[:4])
def test_attention_hd_key_partitions(gpu, dtype, H, G, D, V):
    """Split key ranges: partitions of 32 keys, rows that end before, at and behind their borders."""
    assert _attention_case(gpu, dtype, H, G, D, V, [1] * 6, [1, 31, 32, 33, 97, 200], min_part=32) < TOL[dtype]
    for _ in range(2):  # the tickets re-arm
        assert _attention_case(gpu, dtype, H, G, D, V, [1, 1, 3], [64, 65, 70], min_part=32, seed=7) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,V", [(6, 2, 32, 48), (4, 1, 128, 64), (20, 1, 64, 128)])
def test_attention_hd_one_key_stands_out(gpu, dtype, H, G, D, V):
    assert _attention_case(gpu, dtype, H, G, D, V, [1, 1, 2, 140, 33], [130, 17, 180, 200, 33], spike=True) < TOL[dtype]
    assert _attention_case(gpu, dtype, H, G, D, V, [1, 1, 1], [300, 257, 16], spike=True, min_part=64) < TOL[dtype]


@pytest.mark.parametrize("M,N,K", [(1, 96, 64), (3, 1024, 512), (16, 320, 320), (40, 512, 2048), (100, 96, 192),
                                   (300, 384, 320), (700, 2048, 512), (2049, 2304, 384), (33, 40, 72), (4100, 2560, 1024)])
def test_gemm_relu2_epilogue(gpu, M, N, K):
    """Every row regime of the GEMM planner (GEMV, split-K, ring tiles, ping-pong, four-wave, library)."""
    x, w = rnd(M, K, seed=1, dtype=torch.bfloat16), rnd(N, K, seed=2, dtype=torch.bfloat16, gain=K ** -0.5)
    y = ops.gemm(x.to(gpu), w.to(gpu), epi=ops.EPI_RELU2)
    assert rel_err(y, orc.relu2(x.double() @ w.double().T)) < 1.5e-2
    plain = ops.gemm(x.to(gpu), w.to(gpu))
    assert rel_err(plain, x.double() @ w.double().T) < 1e-2
    z = ops.gemm(x.float().to(gpu), w.float().to(gpu), epi=ops.EPI_RELU2)
    assert rel_err(z, orc.relu2(x.double() @ w.double().T)) < 1e-5


@pytest.mark.parametrize("n,V", [(1, 128256), (3, 150), (200, 9000), (2, 131)])
def test_argmax_fp32_rows(gpu, n, V):
    x = rnd(n, (V + 3) // 4 * 4, seed=4)[:, :V]
    x[:, V // 2] = x[:, 3 * V // 4] = 9.0  # a tie: the lower index
    d = torch.zeros(n, (V + 3) // 4 * 4, device=gpu)
    d[:, :V] = x.to(gpu)
    assert ops.argmax(d[:, :V]).tolist() == [V // 2] * n


def _gla_inputs(step, H, dk, dv, rank, dtype, bias, seed=0):
    nproj = (2 * H * dk + 2 * H * dv + rank + 15) // 16 * 16
    a2, b = rnd(H * dk, rank, seed=seed + 2, dtype=dtype, gain=1.5 / rank ** 0.5), bias + rnd(H * dk, seed=seed + 3)
    return rnd(step.T, nproj, seed=seed + 1, dtype=dtype), a2, b, 1 + rnd(dv, seed=seed + 4, gain=0.2)


def _gla_oracle(x, H, dk, dv, rank, a2, b, nw, tau, eps, state):
    x = x.double()
    T, hk, hv = x.shape[0], H * dk, H * dv
    z = x[:, 2 * hk + 2 * hv:2 * hk + 2 * hv + rank] @ a2.double().T + b.double()
    o, S = orc.gla_recurrence(x[:, :hk].reshape(T, H, dk) * dk ** -0.5, x[:, hk:2 * hk].reshape(T, H, dk),
                              x[:, 2 * hk:2 * hk + hv].reshape(T, H, dv), orc.log_decay(z, tau).reshape(T, H, dk), state)
    o = (orc.rms(o, eps) * nw.double()).reshape(T, hv)
    return o * torch.nn.functional.silu(x[:, 2 * hk + hv:2 * hk + 2 * hv]), S


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dk,dv,rank,tau,bias", [(3, 24, 40, 12, 8.0, 1.0), (2, 32, 64, 16, 16.0, 2.0),
                                                   (1, 100, 30, 5, 1.0, -6.0), (2, 128, 256, 16, 2.0, 0.0),
                                                   (2, 256, 80, 8, 16.0, 3.0), (1, 272, 17, 3, 4.0, 1.0),
                                                   (4, 16, 16, 1, 1.0, -30.0), (2, 8, 129, 20, 3.0, 1.0)])
def test_gla(gpu, dtype, H, dk, dv, rank, tau, bias):
    """Decode rows and portions in one step, starting and continuing sequences, slots that held
    something else before; weak and strong decay (bias)."""
    q_lens, ctx = [1, 1, 2, 15, 16, 17, 64, 65, 150], [1, 40, 2, 80, 16, 17, 64, 165, 150]
    step = Step(q_lens, ctx, gpu, chunk=64)
    eps = 1e-4
    x, a2, b, nw = _gla_inputs(step, H, dk, dv, rank, dtype, bias)
    state = rnd(len(q_lens) + 2, H, dk, dv, seed=9)
    d_state = state.to(gpu)
    out = ops.gla(x.to(gpu), H, dk, dv, a2.to(gpu), b.to(gpu), nw.to(gpu), tau, eps, d_state, step.meta)
    used = set()
    for i, (n, c, s) in enumerate(zip(step.q_lens, step.ctx, step.starts())):
        row = int(step.rows[i])
        used.add(row)
        o, S = _gla_oracle(x[s:s + n], H, dk, dv, rank, a2, b, nw, tau, eps, None if c == n else state[row].double())
        assert rel_err(out[s:s + n], o) < TOL[dtype], (n, c)
        assert rel_err(d_state[row], S) < 3e-5, (n, c)
    for row in set(range(len(state))) - used:
        assert torch.equal(d_state[row].cpu(), state[row])


def test_gla_graph_padding_rows(gpu):
    """Padding rows of a captured decode step (no context) write zeros and touch no state."""
    from mlopamd.runtime.attn_meta import MetaBuffers

    H, dk, dv, rank = 2, 16, 24, 4
    mb = MetaBuffers(8, 8, 4, 16, 2, 64, gpu, flash_min_q=2, flash_tile=128, part_dim=64, chunk=64)
    mb.bt_h[1, :1] = 1
    mb.fill_decode(np.array([1], np.int32), np.array([1], np.int32), np.zeros(1, np.int64), pad_to=4)
    mb.upload()
    meta = mb.meta(4, 4, 4, 32, 1)
    step = type("S", (), {"T": 4})
    x, a2, b, nw = _gla_inputs(step, H, dk, dv, rank, torch.bfloat16, 1.0)
    state = rnd(4, H, dk, dv, seed=9)
    d_state = state.to(gpu)
    out = ops.gla(x.to(gpu), H, dk, dv, a2.to(gpu), b.to(gpu), nw.to(gpu), 2.0, 1e-4, d_state, meta)
    assert float(out[1:].abs().max()) == 0 and float(out[0].abs().max()) > 0
    assert torch.equal(d_state[[0, 2, 3]].cpu(), state[[0, 2, 3]])


@pytest.mark.parametrize("dtype", DTYPES)
def test_gla_large_step(gpu, dtype):
    """A step large enough for the longer chunks (the state passes through dozens of them)."""
    H, dk, dv, rank, tau, eps = 1, 20, 36, 9, 40.0, 1e-4
    q_lens, ctx = [1, 4000, 99, 130], [30, 4100, 99, 131]
    step = Step(q_lens, ctx, gpu, chunk=64)
    assert step.meta.chunk == 128
    x, a2, b, nw = _gla_inputs(step, H, dk, dv, rank, dtype, 2.0, seed=40)
    state = rnd(len(q_lens) + 2, H, dk, dv, seed=9)
    d_state = state.to(gpu)
    out = ops.gla(x.to(gpu), H, dk, dv, a2.to(gpu), b.to(gpu), nw.to(gpu), tau, eps, d_state, step.meta)
    for n, c, s, row in zip(step.q_lens, step.ctx, step.starts(), step.rows.tolist()):
        o, S = _gla_oracle(x[s:s + n], H, dk, dv, rank, a2, b, nw, tau, eps, None if c == n else state[row].double())
        assert rel_err(out[s:s + n], o) < TOL[dtype], (n, c)
        assert rel_err(d_state[row], S) < 5e-5, (n, c)


@pytest.mark.parametrize("dtype", DTYPES)
def test_attention_hd_long_context(gpu, dtype):
    """Hundreds of pages: prompts over many tiles, decode over many partitions, far keys that stand out."""
    assert _attention_case(gpu, dtype, 2, 1, 64, 48, [1, 700, 1], [1500, 1200, 1025], spike=True, min_part=128) < TOL[dtype]
    assert _attention_case(gpu, dtype, 2, 2, 96, 64, [1, 300], [900, 1000]) < TOL[dtype]
