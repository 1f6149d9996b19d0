"""The HIP kernels behind Nafazen's mechanisms (mixers.h, moe.hip, the GEMM epilogues), one by one, against the
plain oracle (tests/nafazen_oracle.py) in fp64 on the same rounded operands, in both element types."""
import pytest
import torch

import nafazen_cases as cases
import nafazen_oracle as orc
from hybrid_util import Step, rel_err
from mlopamd import ops
from mlopamd.models.config import RotarySpec, YarnSpec
from mlopamd.models.layers import rotary_table
from mlopamd.runtime.kv_cache import BLOCK_SIZE, pad_dim

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 2e-5, torch.bfloat16: 1.2e-2}


def rnd(*shape, seed=0, dtype=torch.float32, gain=1.0, mean=0.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * gain + mean).to(dtype)


def up8(n):
    return -(-n // 8) * 8


def rotation(dims, yarn=True, n=2048):
    """(table on the CPU, the oracle's configuration)."""
    rot = {"base": 300.0, "dims": dims, **({"scaling": cases.YARN} if yarn else {})}
    y = cases.YARN
    spec = RotarySpec(300.0, dims, YarnSpec(y["factor"], y["original"], y["fast"], y["slow"]) if yarn else None)
    return rotary_table(spec, n), rot


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W,pad,top", [(1, 64, 0, 1), (5, 72, 56, 2), (300, 1000, 24, 3), (270, 4096, 0, 2), (9, 8150, 42, 1),
                                         (3, 75, 0, 5)])
def test_residual_behind_norms(gpu, dtype, T, W, pad, top):
    """One number per norm, no norm ahead, rows padded with zeros, and a token's expert rows summed."""
    eps, P = 1e-3, W + pad
    padded = lambda t: torch.nn.functional.pad(t, (0, pad)).to(gpu)  # noqa: E731
    table = rnd(40, W, seed=1, dtype=dtype)
    ids = torch.randint(0, 40, (T,), generator=torch.Generator().manual_seed(2))
    pos = torch.zeros(T, dtype=torch.int32, device=gpu)
    g1, g2 = torch.tensor([0.83]), torch.tensor([1.21])
    x, xn = ops.residual_begin(ids.to(gpu), padded(table), 1.7, None, pos, None, eps, width=W)
    ref = 1.7 * table[ids].double()
    assert rel_err(x[:, :W], ref) < 1e-6 and torch.equal(xn, x.to(dtype))
    for k in range(4):
        y = rnd(T, W, seed=20 + k, dtype=dtype, gain=3.0)
        out, kw = y.double(), {}
        if k:  # experts beside a gated shared one, ungated, and alone
            rows = rnd(T * top, W, seed=30 + k, dtype=dtype)
            inv = torch.randperm(T * top, generator=torch.Generator().manual_seed(k)).view(T, top)
            gate = torch.sigmoid(rnd(T, seed=40 + k)) if k == 1 else None
            out = out * gate.double()[:, None] if k == 1 else out if k == 2 else 0
            out = out + rows.double()[inv].sum(1)
            kw = {"experts": (padded(rows), inv.to(torch.int32).to(gpu), None if gate is None else gate.to(gpu))}
        ref = ref + orc.scalar_norm(out, g1.double(), eps)
        last = k == 3
        xn = ops.residual_step(x, None if last else padded(y), g1.to(gpu), g2.to(gpu) if last else None, eps, width=W, **kw)
        assert rel_err(x[:, :W], ref) < 4e-6 and (not pad or float(x[:, W:].abs().max()) == 0)
        assert rel_err(xn[:, :W], orc.scalar_norm(ref, g2.double(), eps) if last else ref) < TOL[dtype]
    assert xn.shape == (T, P)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("R,rot,q,yarn", [(64, 32, 96, True), (44, 12, 36, False), (130, 6, 21, True), (512, 64, 1536, True),
                                          (7, 2, 8, False), (72, 200, 640, False)])
def test_latent_store_with_rotated_keys(gpu, dtype, R, rot, q, yarn):
    """Both norms, the rotation and the paged store of one launch; queries alone."""
    eps = 1e-3
    table, rc = rotation(rot, yarn)
    step = Step([1, 40, 2], [33, 1060, 19], gpu)
    QP, off = pad_dim(q), up8(R)
    proj = rnd(step.T, up8(QP + off + rot), seed=1, dtype=dtype)
    w, qw = rnd(R, seed=2, mean=1.0), rnd(q, seed=3, mean=1.0)
    cache = torch.zeros(step.num_blocks, 1, BLOCK_SIZE, pad_dim(off + rot), dtype=dtype, device=gpu)
    slots = step.meta.slots.clone()
    slots[0] = -1  # a padding row
    pd = proj.to(gpu)
    rope = (pd[:, QP + off:QP + off + rot], table.to(gpu), step.meta.positions, off)
    c_q = ops.latent_store(pd[:, QP:QP + R], w.to(gpu), eps, slots, cache, rope, (pd[:, :q], qw.to(gpu), QP))
    p64, s, pos = proj.double(), step.meta.slots.cpu().long(), step.meta.positions.cpu().tolist()
    got = cache.cpu()[s // BLOCK_SIZE, 0, s % BLOCK_SIZE]
    want = orc.rms(p64[:, QP:QP + R], eps) * w.double()
    turned = torch.cat([orc.rotate(p64[t:t + 1, None, QP + off:QP + off + rot], rc, p)[:, 0] for t, p in enumerate(pos)])
    assert rel_err(got[1:, :R], want[1:]) < TOL[dtype] and float(got[0].abs().max()) == 0
    assert rel_err(got[1:, off:off + rot], turned[1:]) < TOL[dtype]
    assert off == R or float(cache[..., R:off].abs().max()) == 0
    want_q = orc.rms(p64[:, :q], eps) * qw.double()
    for out in (c_q, ops.latent_query(pd[:, :q], qw.to(gpu), QP, eps)):
        assert out.shape == (step.T, QP) and rel_err(out[:, :q], want_q) < TOL[dtype]
        assert q == QP or float(out[:, q:].abs().max()) == 0


def _case(gpu, dtype, H, D, V, R, rot, q_lens, ctx, min_part=None, spike=False, seed=0, yarn=True):
    """Max relative error of a step of latent attention with a rotated part against the oracle.  ``spike``: every
    query asks for one key whose score stands out, by its unrotated part (even heads) or its rotated one (odd):
    the first token, its own, its predecessor, or the other side of a page border."""
    q_off, k_off = up8(D), up8(R)
    KP, RP, KD, VP = pad_dim(q_off + rot), pad_dim(k_off + rot), pad_dim(q_off), pad_dim(V)
    table, rc = rotation(rot, yarn, max(ctx))
    step = Step(q_lens, ctx, gpu, n_kv=-(-H // 16), min_part=min_part, part_dim=RP, seed=seed, expand_window=0)
    scale = 1.7 * (D + rot) ** -0.5
    uk, uv = rnd(H, D, R, seed=seed + 1, dtype=dtype, gain=R ** -0.5), rnd(H, V, R, seed=seed + 2, dtype=dtype, gain=R ** -0.5)
    w_k, w_v = torch.zeros(H, KP, RP, dtype=dtype), torch.zeros(H, VP, RP, dtype=dtype)
    w_k[:, :D, :R], w_v[:, :V, :R] = uk, uv
    w_k[:, q_off:q_off + rot, k_off:k_off + rot] = torch.eye(rot)
    w_qk, w_vo = torch.zeros(H, k_off, KD, dtype=dtype), torch.zeros(H, V, pad_dim(R), dtype=dtype)
    w_qk[:, :R, :D], w_vo[:, :, :R] = uk.transpose(1, 2), uv
    cache = torch.zeros(step.num_blocks, 1, BLOCK_SIZE, RP, dtype=dtype)
    q = torch.zeros(step.T, H, KP, dtype=dtype)
    want = torch.zeros(step.T, H * V, dtype=torch.float64)
    for i, (n, c, s) in enumerate(zip(step.q_lens, step.ctx, step.starts())):
        lat, k_rot = rnd(c, R, seed=seed + 10 + i, dtype=dtype), rnd(c, rot, seed=seed + 30 + i, dtype=dtype)
        k = torch.einsum("tr,hdr->thd", lat.double(), uk.double())
        v = torch.einsum("tr,hvr->thv", lat.double(), uv.double())
        qq, qr = rnd(c, H, D, seed=seed + 50 + i, dtype=dtype), rnd(c, H, rot, seed=seed + 70 + i, dtype=dtype)
        if spike:
            for t in range(c - n, c):
                for h in range(H):
                    j = [0, t, max(0, t - 1), max(0, t - t % 16 - 1)][(t + h // 2) % 4]
                    if h % 2 == 0:
                        qq[t, h] = (k[j, h] * (14.0 / scale / k[j, h].pow(2).sum())).to(dtype)
                    else:  # turned back from the query's own position, it meets the turned key
                        goal = k_rot[j].double() * (14.0 / scale / k_rot[j].double().pow(2).sum())
                        one = orc.rotate(torch.eye(rot, dtype=torch.float64)[None], rc, t)[0]  # rows: turned axes
                        qr[t, h] = (goal @ torch.linalg.inv(one)).to(dtype)
        row = torch.zeros(c, 1, RP, dtype=dtype)
        row[:, 0, :R], row[:, 0, k_off:k_off + rot] = lat, k_rot
        step.scatter(cache, i, row, c)
        q[s:s + n, :, :D], q[s:s + n, :, q_off:q_off + rot] = qq[c - n:], qr[c - n:]
        turned = orc.rotate(qr.double(), rc)
        o = cases.fast_attention(qq.double(), k, v, turned, k_rot.double(), scale)
        want[s:s + n] = o[c - n:].reshape(n, H * V)
    w_kv = torch.cat([w_k.view(H * KP, RP), w_v.view(H * VP, RP)])
    out = ops.latent_attention(q.to(gpu), None, cache.to(gpu), w_kv.to(gpu), w_qk.to(gpu), w_vo.to(gpu), V, scale, 0, None,
                               step.meta, rope=(table.to(gpu), rot, q_off, k_off))
    return max(rel_err(out[s:s + n], want[s:s + n]) for n, s in zip(step.q_lens, step.starts()))


# latent rows of one to nine blocks and past the kernels', odd and even, values in all blocks or all but the last
SIZES = [(6, 32, 48, 128, 32), (3, 20, 28, 44, 12), (20, 64, 128, 512, 64), (16, 128, 64, 256, 64), (1, 200, 250, 330, 26),
         (33, 16, 24, 72, 8), (2, 128, 128, 448, 128), (4, 40, 24, 64, 2), (2, 40, 23, 600, 40), (5, 30, 32, 190, 6)]
# bf16: queries and results pass through the latent space rounded once more
LTOL = {torch.float32: 3e-5, torch.bfloat16: 2.5e-2}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,V,R,rot", SIZES)
def test_rotated_latent_attention(gpu, dtype, H, D, V, R, rot):
    # decoded tokens and portions down to two tokens, contexts at page and tile borders
    q_lens = [1, 1, 1, 1, 1, 1, 2, 3, 31, 130, 17]
    ctx = [1, 16, 17, 24, 65, 161, 2, 67, 31, 150, 48]
    assert _case(gpu, dtype, H, D, V, R, rot, q_lens, ctx) < LTOL[dtype]
    assert _case(gpu, dtype, H, D, V, R, rot, [1, 5], [40, 21], seed=3, yarn=False) < LTOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,V,R,rot", SIZES)
def test_rotated_latent_attention_key_partitions(gpu, dtype, H, D, V, R, rot):
    for seed in (0, 1):
        assert _case(gpu, dtype, H, D, V, R, rot, [1] * 6, [1, 129, 300, 33, 97, 520], min_part=32, seed=seed) < LTOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,V,R,rot", [SIZES[0], SIZES[4], SIZES[5]])
def test_rotated_latent_attention_one_key_stands_out(gpu, dtype, H, D, V, R, rot):
    assert _case(gpu, dtype, H, D, V, R, rot, [1, 1, 1, 2, 140, 33], [130, 17, 51, 180, 200, 33], spike=True) < 2 * LTOL[dtype]
    assert _case(gpu, dtype, H, D, V, R, rot, [1, 1, 1], [900, 257, 16], spike=True, min_part=64) < 2 * LTOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_rotated_latent_attention_long_context(gpu, dtype):
    assert _case(gpu, dtype, 2, 64, 48, 96, 32, [1, 300, 1], [1500, 1400, 1025], spike=True) < 2 * LTOL[dtype]


def test_graph_padding_rows_get_zeros(gpu):
    """Padding rows of a decode bucket: no key, no store, zeros."""
    import numpy as np

    from mlopamd.runtime.attn_meta import MetaBuffers

    mb = MetaBuffers(8, 8, 4, 16, 1, 64, gpu, flash_min_q=2, flash_tile=128, part_dim=128, chunk=64, expand_window=0)
    mb.bt_h[2, :2] = [1, 2]
    mb.fill_decode(np.array([2], np.int32), np.array([20], np.int32), np.zeros(1, np.int64), pad_to=4)
    mb.upload()
    meta = mb.meta(4, 4, 4, 32, 1)
    cache = rnd(4, 1, 16, 128, seed=1, dtype=torch.bfloat16).to(gpu)
    q = rnd(4, 2, 64, seed=2, dtype=torch.bfloat16).to(gpu)
    table = rotation(8)[0].to(gpu)
    w = lambda *s: rnd(*s, seed=3, dtype=torch.bfloat16, gain=0.1).to(gpu)  # noqa: E731
    out = ops.latent_attention(q, None, cache, w(2 * 128, 128), w(2, 72, 64), w(2, 24, 128), 24, 0.2, 0, None, meta,
                               rope=(table, 8, 24, 72))
    assert float(out[1:].abs().max()) == 0 and float(out[0].abs().max()) > 0


@pytest.mark.parametrize("M,N,K", [(1, 64, 64), (3, 512, 512), (8, 1024, 1024), (16, 160, 320), (40, 256, 2048), (100, 96, 192),
                                   (200, 512, 1024), (300, 640, 512), (1100, 1024, 256), (2048, 6144, 256), (2100, 512, 4096)])
def test_gemm_xielu(gpu, M, N, K):
    x, w = rnd(M, K, seed=1, dtype=torch.bfloat16), rnd(N, K, seed=2, dtype=torch.bfloat16, gain=2 * K ** -0.5)
    p, q = torch.tensor(0.4, dtype=torch.float64), torch.tensor(-0.9, dtype=torch.float64)
    a, b = orc.softplus(p).item(), 0.5 + orc.softplus(q).item()
    z = x.double().to(gpu) @ w.double().to(gpu).T
    want = orc.xielu(z, p.to(gpu), q.to(gpu))
    assert rel_err(ops.gemm(x.to(gpu), w.to(gpu), epi=ops.EPI_XIELU, xielu=(a, b)), want) < 6e-3
    neg = z < -0.5  # where the result is small beside the largest
    got = ops.gemm(x.to(gpu), w.to(gpu), epi=ops.EPI_XIELU, xielu=(a, b)).double()
    assert float(((got - want).abs() / want.abs().clamp_min(0.05))[neg].max()) < 2e-2
    f = ops.gemm(x.float().to(gpu), w.float().to(gpu), epi=ops.EPI_XIELU, xielu=(a, b))
    assert rel_err(f, want) < 1e-5
    assert rel_err(ops.xielu(z.float().contiguous(), a, b), want) < 1e-6


def _router(E, gated, W, seed):
    """Tokens and router rows without close calls: every token leans to the experts it will choose."""
    g = torch.Generator().manual_seed(seed)
    axes = torch.linalg.qr(torch.randn(W, max(E + 1, 1), generator=g))[0].T
    w = (0.1 * axes[:E + gated]).to(torch.bfloat16)

    def tokens(T, top):
        x = torch.randn(T, W, generator=g)
        lean = torch.zeros(T, E).scatter(1, torch.argsort(torch.rand(T, E, generator=g), 1)[:, :top], 12.0 + torch.rand(T, top, generator=g) * 9)
        return (x + lean @ axes[:E]).to(torch.bfloat16)
    return w, tokens


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,top,gated,W", [(5, 2, True, 128), (1, 1, True, 192), (12, 1, False, 1024), (8, 2, True, 4096), (40, 40, True, 320),
                                           (200, 6, True, 2048), (16, 3, False, 1000)])
def test_sigmoid_routing_and_experts(gpu, dtype, E, top, gated, W):
    """Choice, scores, gates, sorted rows; and the experts' gated unit on inputs times their scores, through the
    gathered rows (few tokens) and in place (many)."""
    if W % 64 and dtype == torch.bfloat16:
        experts = False  # (the grouped product takes whole tiles of 64)
    else:
        experts = E <= 16
    w, tokens = _router(E, gated, W, seed=E)
    I = 96
    w13, w2 = rnd(E, 2 * I, W, seed=3, dtype=torch.bfloat16, gain=W ** -0.5) if experts else None, None
    for T in (1, 2, 16, 17, 70, 600, 2100) if E < 100 else (3, 40):
        x = tokens(T, top)
        d = ops.moe_dispatch_input(x.to(gpu, dtype), w.to(gpu, dtype), E, top)
        z = x.double() @ w.double().T
        off, inv = d.offsets.tolist(), d.inv.cpu()
        assert off[-1] == T * top and sorted(inv.flatten().tolist()) == list(range(T * top))
        expert_of = torch.bucketize(inv, d.offsets.cpu()[1:], right=True)
        best, s = torch.sort(torch.topk(z[:, :E], top, -1).indices, -1).values, torch.sigmoid(z[:, :E])
        assert torch.equal(torch.sort(expert_of, -1).values, best)
        assert (d.gate is not None) == gated and (not gated or rel_err(d.gate, torch.sigmoid(z[:, E])) < 1e-5)
        score = torch.gather(s, 1, expert_of)
        if d.a_rows is None:
            assert rel_err(d.x.cpu()[inv.long()], score[..., None] * x.double()[:, None]) < (5e-3 if dtype == torch.bfloat16 else 1e-5)
        else:
            assert torch.equal(d.a_rows.cpu()[inv.long()], torch.arange(T, dtype=torch.int32)[:, None].expand(T, top))
            assert rel_err(d.row_w.cpu()[inv.long()], score) < 1e-5
        if experts:
            got = ops.grouped_gemm(d.x, w13.to(gpu, dtype), d.offsets, epi=ops.EPI_SILU_MUL, avg_rows=max(1, T * top // E),
                                   a_rows=d.a_rows, row_scale=d.row_w).cpu()[inv.long()]
            gu = ops.deinterleave_cols(torch.einsum("tk,ekn->ten", x.double(), w13.double().transpose(1, 2)))
            gu = torch.gather(gu, 1, expert_of[..., None].expand(T, top, 2 * I)) * score[..., None]
            want = orc.silu(gu[..., :I]) * gu[..., I:]
            assert rel_err(got, want) < (1.5e-2 if dtype == torch.bfloat16 else 2e-5), T


@pytest.mark.parametrize("avg", [1, 8, 30, 60, 120, 250, 700])
@pytest.mark.parametrize("N,K,E", [(512, 64, 3), (1024, 2048, 2), (96, 128, 7), (256, 192, 4)])
def test_grouped_rows_scaled_in_place(gpu, avg, N, K, E):
    """Row scales in every tile shape the planner has for a row count (also split K ranges)."""
    T = avg * E // 2 + 17
    g = torch.Generator().manual_seed(avg)
    x, w = rnd(T, K, seed=1, dtype=torch.bfloat16), rnd(E, N, K, seed=2, dtype=torch.bfloat16, gain=2 * K ** -0.5)
    expert = torch.sort(torch.randint(0, E, (2 * T,), generator=g)).values
    offsets = torch.searchsorted(expert, torch.arange(E + 1)).to(torch.int32)
    rows = torch.randint(0, T, (2 * T,), generator=g).to(torch.int32)
    sc = torch.rand(2 * T, generator=g) * 2
    got = ops.grouped_gemm(x.to(gpu), w.to(gpu), offsets.to(gpu), epi=ops.EPI_SILU_MUL, avg_rows=avg, a_rows=rows.to(gpu),
                           row_scale=sc.to(gpu))
    xs = x.double()[rows.long()] * sc.double()[:, None]
    want = torch.cat([ops.deinterleave_cols(xs[a:b] @ w[e].double().T) for e, (a, b) in enumerate(zip(offsets, offsets[1:]))])
    want = orc.silu(want[:, :N // 2]) * want[:, N // 2:]
    assert rel_err(got, want) < 1.5e-2


@pytest.mark.parametrize("R,N,K,G", [(1, 64, 64, 1), (77, 96, 200, 5), (300, 130, 33, 3)])
def test_grouped_plain(gpu, R, N, K, G):
    x, w = rnd(R, K, seed=1), rnd(G, N, K, seed=2, gain=K ** -0.5)
    cut = sorted([0, R, *torch.randint(0, R + 1, (G - 1,), generator=torch.Generator().manual_seed(3)).tolist()])
    got = ops.grouped_gemm(x.to(gpu), w.to(gpu), torch.tensor(cut, dtype=torch.int32, device=gpu))
    want = torch.cat([x[a:b].double() @ w[e].double().T for e, (a, b) in enumerate(zip(cut, cut[1:]))])
    assert rel_err(got, want) < 1e-5
