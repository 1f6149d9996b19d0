"""The HIP kernels behind Dibedra's mechanisms (hybrid.h, mixers.h, moe.hip, the GEMM epilogues), one by one, against
the plain oracle (tests/dibedra_oracle.py) in fp64 on the same rounded operands, in both element types."""
import pytest
import torch

import dibedra_cases as cases
import dibedra_oracle as orc
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


def rotation(dims, yarn=True, n=2048):
    """(table on the CPU, the oracle's configuration)."""
    rot = {"base": 300.0, "dims": dims, **({"scaling": cases.YARN} if yarn else {})}
    y = cases.YARN
    spec = RotarySpec(300.0, dims, YarnSpec(y["factor"], y["original"], y["fast"], y["slow"]) if yarn else None)
    return rotary_table(spec, n), rot


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W,pad,top", [(1, 64, 0, 1), (5, 72, 56, 2), (300, 1000, 24, 3), (270, 4096, 0, 3), (9, 8150, 42, 1),
                                         (3, 75, 0, 5)])
def test_dynamic_tanh_residual(gpu, dtype, T, W, pad, top):
    """The norm ahead of the next layer, and both sublayers' outputs added in the pass: attention's row, expert rows
    with their weights (some of the token's choices without a row), the token's own input."""
    padded = lambda t: torch.nn.functional.pad(t, (0, pad)).to(gpu)  # noqa: E731
    g = torch.Generator().manual_seed(T)
    table, w, b = rnd(40, W, seed=1, dtype=dtype), rnd(W, seed=2, mean=1.2, gain=0.3), rnd(W, seed=3, gain=0.3)
    ids = torch.randint(0, 40, (T,), generator=g)
    pos, alpha = torch.zeros(T, dtype=torch.int32, device=gpu), torch.tensor([0.37])
    norm = {"norm_w": padded(w), "eps": 0.0, "tanh": (alpha.to(gpu), padded(b))}
    x, h = ops.residual_begin(ids.to(gpu), padded(table), 1.0, None, pos, **norm)
    ref = table[ids].double()
    tanh = lambda v: orc.dynamic_tanh(v, alpha.double(), w.double(), b.double())  # noqa: E731
    assert rel_err(x[:, :W], ref) < 1e-6 and rel_err(h[:, :W], tanh(ref)) < (2e-6 if dtype == torch.float32 else 5e-3)
    for k in range(5):
        y = rnd(T, W, seed=20 + k, dtype=dtype, gain=2.0)
        out, kw = y.double(), {}
        if k:  # with the token itself, without it, no weights, nothing but experts
            rows, weight = rnd(T * top, W, seed=30 + k, dtype=dtype), torch.rand(T, top, generator=g)
            inv = torch.randperm(T * top, generator=g).view(T, top)
            inv[torch.rand(T, top, generator=g) < 0.3] = -1
            own = torch.rand(T, generator=g) * (torch.rand(T, generator=g) < 0.6)
            kw = {"experts": (padded(rows), inv.to(torch.int32).to(gpu), None)}
            part = rows.double()[inv.clamp(min=0)] * (inv >= 0)[..., None]
            if k == 3:
                part = part.sum(1)
            else:
                kw["share"] = (weight.to(gpu), h if k == 1 else None, own.to(gpu) if k == 1 else None)
                part = (part * weight.double()[..., None]).sum(1)
            if k == 1:
                part = part + own.double()[:, None] * h[:, :W].double().cpu()
            out = out + part if k < 4 else part
        ref = ref + out
        h = ops.residual_step(x, None if k == 4 else padded(y), None, **norm, **kw)
        assert rel_err(x[:, :W], ref) < 4e-6 and (not pad or float(x[:, W:].abs().max()) == 0)
        assert rel_err(h[:, :W], tanh(ref)) < (2e-6 if dtype == torch.float32 else 5e-3)
        assert not pad or float(h[:, W:].abs().max()) == 0


def test_dynamic_tanh_of_all_sizes(gpu):
    """From tiny arguments to saturated ones."""
    v = torch.cat([10.0 ** torch.arange(-7, 3, 0.125), torch.zeros(4), torch.linspace(0.1, 1.0, 172)])
    table = torch.stack([v, -v])
    one, zero = torch.ones(v.numel()), torch.zeros(v.numel())
    _, h = ops.residual_begin(torch.arange(2, device=gpu), table.to(gpu), 1.0, None, torch.zeros(2, dtype=torch.int32, device=gpu),
                              one.to(gpu), 0.0, tanh=(torch.tensor([0.7], device=gpu), zero.to(gpu)))
    want = torch.tanh(torch.tensor([0.7]).double() * table.double())
    assert float(((h.double().cpu() - want).abs() / want.abs().clamp_min(1e-30)).max()) < 1e-6


HEADS = [(4, 2, 64, 64), (6, 2, 20, 12), (3, 1, 34, 34), (8, 8, 128, 128), (5, 5, 200, 136), (2, 1, 328, 64), (36, 2, 24, 8), (7, 7, 8, 2),
         (32, 8, 128, 96), (3, 3, 9, 4), (2, 2, 600, 64), (1, 1, 72, 0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,R", HEADS)
def test_per_head_norm(gpu, dtype, H, G, D, R):
    """Norm, rotation and the paged stores; values the keys as given, or columns of their own."""
    eps = 1e-2
    table, rot = (torch.zeros(2048, 0), None) if R == 0 else rotation(R, yarn=H % 2 == 0)
    step = Step([1, 40, 2, 1500] if H == 32 else [1, 40, 2], [33, 1060, 19, 1500] if H == 32 else [33, 1060, 19], gpu)
    up8 = lambda n: -(-n // 8) * 8  # noqa: E731
    for V in (0, max(1, D - 7)):
        k0, v0, end = up8(H * D) + 8, up8(H * D) + 8 + up8(G * D), up8(H * D) + 16 + up8(G * D) + up8(G * V)
        proj = rnd(step.T, end, seed=1, dtype=dtype).to(gpu)
        q, k, v = proj[:, :H * D], proj[:, k0:k0 + G * D], proj[:, v0:v0 + G * V] if V else None
        qw, kw = rnd(D, seed=2, mean=1.0, gain=0.3), rnd(D, seed=3, mean=1.0, gain=0.3)
        kc = torch.zeros(step.num_blocks, G, BLOCK_SIZE, pad_dim(D), dtype=dtype, device=gpu)
        vc = torch.zeros(step.num_blocks, G, BLOCK_SIZE, pad_dim(V or D), dtype=dtype, device=gpu)
        slots = step.meta.slots.clone()
        slots[0] = -1  # a padding row
        out = ops.qk_head_norm(q, k, v, H, D, V or D, qw.to(gpu), kw.to(gpu), eps, table.to(gpu), step.meta.positions, slots, kc, vc)
        s = step.meta.slots.cpu().long()

        def turned(x, heads, w):
            x = orc.head_norm(x.double().cpu().reshape(-1, heads, D), w.double(), eps)
            return x if R == 0 else torch.cat([orc.rotate(x[s:s + n], rot, c - n) for s, n, c in zip(step.starts(), step.q_lens, step.ctx)])

        assert out.shape == (step.T, H, pad_dim(D)) and rel_err(out[..., :D], turned(q, H, qw)) < TOL[dtype]
        assert D % 64 == 0 or float(out[..., D:].abs().max()) == 0
        got_k, got_v = (c.cpu()[s // BLOCK_SIZE, :, s % BLOCK_SIZE] for c in (kc, vc))
        assert rel_err(got_k[1:, :, :D], turned(k, G, kw)[1:]) < TOL[dtype] and float(got_k[0].abs().max()) == 0
        assert torch.equal(got_v[1:, :, :V or D], (k if v is None else v).cpu().reshape(-1, G, V or D)[1:])
        assert float(got_v[0].abs().max()) == 0 and (D % 64 == 0 or float(kc[..., D:].abs().max()) == 0)


def _case(gpu, dtype, H, G, D, window, q_lens, ctx, min_part=None, spike=False, seed=0):
    """Max relative error of a step of windowed, gated attention into columns of a wider row, against the oracle.
    ``spike``: every query asks for one key whose score stands out: its own, the last one inside the window, the first
    one outside, the first token, or the other side of a page border."""
    step = Step(q_lens, ctx, gpu, n_kv=G * -(-(H // G) // 16), min_part=min_part, part_dim=pad_dim(D), seed=seed)
    KP, scale, T = pad_dim(D), 1.3 * D ** -0.5, step.T
    kc, vc = (torch.zeros(step.num_blocks, G, BLOCK_SIZE, KP, dtype=dtype) for _ in range(2))
    q, want = torch.zeros(T, H, KP, dtype=dtype), torch.zeros(T, H * D, dtype=torch.float64)
    gate = rnd(T, H * D + 24, seed=seed + 5, dtype=dtype, gain=2.0)
    for i, (n, c, s) in enumerate(zip(step.q_lens, step.ctx, step.starts())):
        k, v = rnd(c, G, D, seed=seed + 10 + i, dtype=dtype), rnd(c, G, D, seed=seed + 30 + i, dtype=dtype)
        qq = rnd(c, H, D, seed=seed + 50 + i, dtype=dtype)
        if spike:
            for t in range(c - n, c):
                for h in range(H):
                    j = [t, max(0, t - window + 1), max(0, t - window), 0, max(0, t - t % 16 - 1)][(t + h) % 5]
                    goal = k[j, h // (H // G)].double()
                    qq[t, h] = (goal * (14.0 / scale / goal.pow(2).sum())).to(dtype)
        step.scatter(kc, i, k, c)
        step.scatter(vc, i, v, c)
        q[s:s + n, :, :D] = qq[c - n:]
        o = cases.fast_attention(qq.double(), k.double(), v.double(), scale, window)[c - n:].reshape(n, H * D)
        want[s:s + n] = orc.output_gate(o, gate[s:s + n, 8:8 + H * D].double())
    row = torch.full((T, 64 + -(-H * D // 8) * 8), 7.0, dtype=dtype, device=gpu)
    ops.attention_hd(q.to(gpu), kc.to(gpu), vc.to(gpu), step.meta, D, D, scale, gate=gate.to(gpu)[:, 8:8 + H * D], window=window,
                     out=row[:, 8:8 + H * D].unflatten(1, (H, D)))
    assert float((row[:, :8] - 7).abs().max()) == 0 and float((row[:, 8 + H * D:] - 7).abs().max()) == 0
    got = row[:, 8:8 + H * D]
    return max(rel_err(got[s:s + n], want[s:s + n]) for n, s in zip(step.q_lens, step.starts()))


SIZES = [(6, 2, 64), (6, 2, 20), (7, 1, 34), (8, 8, 128), (3, 3, 200), (2, 1, 328), (36, 2, 24), (20, 1, 128), (4, 4, 256), (3, 1, 9)]
ATOL = {torch.float32: 3e-5, torch.bfloat16: 1.5e-2}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [0, 1, 2, 16, 17, 33, 96, 129])
@pytest.mark.parametrize("H,G,D", SIZES)
def test_windowed_attention(gpu, dtype, H, G, D, window):
    # decoded tokens and portions down to two tokens, contexts at page, tile and window borders
    q_lens = [1, 1, 1, 1, 1, 1, 2, 3, 31, 130, 17]
    ctx = [1, 16, 17, 33, 97, 161, 2, 67, 31, 250, 48]
    assert _case(gpu, dtype, H, G, D, window, q_lens, ctx) < ATOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [0, 5, 100])
@pytest.mark.parametrize("H,G,D", SIZES)
def test_windowed_attention_key_partitions(gpu, dtype, H, G, D, window):
    for seed in (0, 1):
        assert _case(gpu, dtype, H, G, D, window, [1] * 6, [1, 129, 300, 33, 97, 520], min_part=32, seed=seed) < ATOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [1, 2, 16, 17, 64, 100])
@pytest.mark.parametrize("H,G,D", [SIZES[0], SIZES[1], SIZES[3], SIZES[7]])
def test_one_key_stands_out(gpu, dtype, H, G, D, window):
    assert _case(gpu, dtype, H, G, D, window, [1, 1, 1, 2, 140, 33], [130, 17, 51, 180, 300, 33], spike=True) < 2 * ATOL[dtype]
    assert _case(gpu, dtype, H, G, D, window, [1, 1, 1], [900, 257, 16], spike=True, min_part=64) < 2 * ATOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_windowed_attention_long_context(gpu, dtype):
    for window in (0, 1024, 700):
        assert _case(gpu, dtype, 4, 2, 64, window, [1, 300, 1], [1500, 1400, 1025], spike=window > 0) < 2 * ATOL[dtype]


def test_graph_padding_rows_get_zeros(gpu):
    """Padding rows of a decode bucket: no key, zeros, also where the output is columns of a wider row."""
    import numpy as np

    from mlopamd.runtime.attn_meta import MetaBuffers

    mb = MetaBuffers(8, 8, 4, 16, 2, 64, gpu, flash_min_q=2, flash_tile=128, part_dim=64, chunk=0)
    mb.bt_h[2, :2] = [1, 2]
    mb.fill_decode(np.array([2], np.int32), np.array([20], np.int32), np.zeros(1, np.int64), pad_to=4)
    mb.upload()
    cache = rnd(4, 2, 16, 64, seed=1, dtype=torch.bfloat16).to(gpu)
    q, row = rnd(4, 4, 64, seed=2, dtype=torch.bfloat16).to(gpu), torch.full((4, 256), 7.0, dtype=torch.bfloat16, device=gpu)
    for part, nparts in ((64, 1), (32, 2)):
        ops.attention_hd(q, cache, cache, mb.meta(4, 4, 4, part, nparts), 40, 40, 0.2, gate=row[:, 64:224], window=9,
                         out=row[:, :160].unflatten(1, (4, 40)))
        assert float(row[1:, :160].abs().max()) == 0 and float(row[0, :160].abs().max()) > 0 and float((row[:, 224:] - 7).abs().max()) == 0
        row[:, :160] = 7


@pytest.mark.parametrize("M,N,K", [(1, 64, 64), (3, 512, 512), (4, 1024, 1024), (16, 192, 320), (40, 256, 2048), (100, 448, 192),
                                   (200, 512, 1024), (300, 640, 512), (1100, 1024, 256), (2048, 6144, 256), (2100, 512, 4096)])
def test_gemm_gelu(gpu, M, N, K):
    """The activation on all columns, and from a column on; a product over columns of a wider row."""
    x, w = rnd(M, K + 128, seed=1, dtype=torch.bfloat16), rnd(N, K, seed=2, dtype=torch.bfloat16, gain=2 * K ** -0.5)
    xg = x.to(gpu)[:, 64:64 + K]
    z = xg.double() @ w.double().to(gpu).T
    for n0 in {0, min(128, N // 128 * 128), N // 2 // 128 * 128, (N - 1) // 128 * 128}:
        want = torch.cat([z[:, :n0], orc.gelu_tanh(z[:, n0:])], 1)
        got = ops.gemm(xg, w.to(gpu), epi=ops.EPI_GELU, act_from=n0).double()
        assert rel_err(got, want) < 6e-3
        neg = z < -0.5  # where the result is small beside the largest
        neg[:, :n0] = False
        assert not neg.any() or float(((got - want).abs() / want.abs().clamp_min(0.01))[neg].max()) < 2e-2
        f = ops.gemm(xg.float(), w.float().to(gpu), epi=ops.EPI_GELU, act_from=n0)
        assert rel_err(f, want) < 1e-5
    assert rel_err(ops.gelu_tanh(z.float().contiguous()), orc.gelu_tanh(z)) < 1e-6


@pytest.mark.parametrize("n0", [0, 128, 256])
def test_other_activations_from_a_column_on(gpu, n0):
    x, w = rnd(70, 128, seed=1, dtype=torch.bfloat16).to(gpu), rnd(320, 128, seed=2, dtype=torch.bfloat16, gain=0.2).to(gpu)
    z = x.double() @ w.double().T
    for dtype, tol in ((torch.bfloat16, 6e-3), (torch.float32, 1e-5)):
        got = ops.gemm(x.to(dtype), w.to(dtype), epi=ops.EPI_RELU2, act_from=n0)
        assert rel_err(got, torch.cat([z[:, :n0], z[:, n0:].clamp(min=0) ** 2], 1)) < tol


# (experts, identity experts, chosen, groups, kept, width)
ROUTES = [(5, 2, 3, 1, 1, 128), (1, 0, 1, 1, 1, 192), (9, 0, 9, 3, 3, 64), (12, 3, 4, 5, 2, 1024), (1, 7, 2, 2, 2, 72), (8, 4, 3, 3, 2, 4096),
          (6, 6, 12, 1, 1, 320), (40, 8, 6, 4, 1, 384), (16, 8, 3, 6, 3, 2048), (250, 6, 24, 16, 5, 256), (90, 10, 7, 5, 2, 2048), (63, 1, 20, 64, 40, 1000), (3, 5, 2, 8, 3, 8192)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,identity,top,groups,keep,W", ROUTES)
def test_grouped_routing(gpu, dtype, E, identity, top, groups, keep, W):
    """Scores, the choice of groups and of outputs in them, sorted rows; identity experts have a weight and no row."""
    n = E + identity
    g = torch.Generator().manual_seed(n)
    router = (2.0 * torch.randn(n, W, generator=g) * W ** -0.5).to(torch.bfloat16)
    corr = 0.3 * torch.randn(n, generator=g)
    for correction in (corr, None):
        for T in (1, 2, 16, 17, 70, 600, 2100) if correction is corr and n < 100 else (3, 40, 1100):
            x = torch.randn(T, W, generator=g).to(torch.bfloat16)
            d = ops.moe_dispatch_groups(x.to(gpu, dtype), router.to(gpu, dtype), None if correction is None else corr.to(gpu), E, top,
                                        groups, keep)
            z = x.double() @ router.double().T
            off, inv, top_w = d.offsets.tolist(), d.inv.cpu(), d.top_w.cpu().double()
            real = inv >= 0
            assert off[-1] == int(real.sum()) and sorted(inv[real].tolist()) == list(range(off[-1]))
            expert_of = torch.bucketize(inv, d.offsets.cpu()[1:], right=True)
            assert (d.self_w is None) == (identity == 0)
            for t in range(0, T, max(1, T // 150)):
                c = (corr if correction is corr else 0 * corr).double()
                choice = orc.softmax_scores(z[t]) + c
                want = dict(orc.choose(z[t], c, groups, keep, top))
                best = choice.view(groups, -1).max(-1).values.sort(descending=True).values
                inside = torch.stack(sorted((choice[i] for i in orc.best_groups(choice, groups, keep)), reverse=True))
                if (keep < groups and best[keep - 1] - best[keep] < 1e-5) or (len(inside) > top and inside[top - 1] - inside[top] < 1e-5):
                    continue  # a tie
                got = {int(e): float(s) for e, s, r in zip(expert_of[t], top_w[t], real[t]) if r}
                assert got.keys() == {e for e in want if e < E}, t
                assert all(abs(s - float(want[e])) < 1e-5 for e, s in got.items())
                own = sum(float(s) for e, s in want.items() if e >= E)
                assert identity == 0 or abs(float(d.self_w[t]) - own) < 1e-5
            rows = d.x.cpu() if d.a_rows is None else d.x.cpu()[d.a_rows.cpu().long().clamp(0, T - 1)]
            at, tok = inv[real].long(), torch.arange(T)[:, None].expand(T, top)[real]
            assert torch.equal(rows[at], x.to(dtype)[tok])


def test_ties_go_to_the_first(gpu):
    """Equal choice scores: the lower output and the lower group win, whatever the lane that holds them."""
    x = torch.ones(20, 64, dtype=torch.bfloat16, device=gpu)
    for T in (3, 20):
        d = ops.moe_dispatch_groups(x[:T], torch.zeros(200, 64, dtype=torch.bfloat16, device=gpu), None, 200, 5, 50, 2)
        assert d.offsets.tolist()[:9] == [0, T, 2 * T, 3 * T, 4 * T, 5 * T, 5 * T, 5 * T, 5 * T]
        assert rel_err(d.top_w, torch.full((T, 5), 1 / 200)) < 1e-6


@pytest.mark.parametrize("avg", [1, 2, 8, 30, 60, 120, 250, 700])
@pytest.mark.parametrize("N,K,E", [(512, 64, 3), (1024, 2048, 2), (128, 128, 7), (256, 192, 4)])
def test_grouped_clamped_unit(gpu, avg, N, K, E):
    """The experts' unit in every tile shape the planner has for a row count (also split K ranges), over gathered rows
    and in place, with rows that belong to no expert behind the last one."""
    T = avg * E // 2 + 2
    g = torch.Generator().manual_seed(avg)
    x, w = rnd(T, K, seed=1, dtype=torch.bfloat16), rnd(E, N, K, seed=2, dtype=torch.bfloat16, gain=2 * K ** -0.5)
    expert = torch.sort(torch.randint(0, E, (2 * T,), generator=g)).values
    used = 2 * T - 1
    offsets = torch.searchsorted(expert[:used], torch.arange(E + 1)).to(torch.int32)
    rows = torch.randint(0, T, (2 * T,), generator=g).to(torch.int32)
    want = torch.cat([ops.deinterleave_cols(x.double()[rows[a:b].long()] @ w[e].double().T) for e, (a, b) in enumerate(zip(offsets, offsets[1:]))])
    want = orc.clamped_unit(want[:, :N // 2], want[:, N // 2:], 1.3)
    glu = dict(epi=ops.EPI_SILU_MUL, glu=(1.702, 1.3))
    rows[used:] = 0
    got = ops.grouped_gemm(x.to(gpu), w.to(gpu), offsets.to(gpu), avg_rows=avg, a_rows=rows.to(gpu), **glu)
    assert rel_err(got[:used], want) < 1e-2
    xp = x[rows.long()]
    assert rel_err(ops.grouped_gemm(xp.to(gpu), w.to(gpu), offsets.to(gpu), avg_rows=avg, **glu)[:used], want) < 1e-2
    if T < 600:
        assert rel_err(ops.grouped_gemm(xp.float().to(gpu), w.float().to(gpu), offsets.to(gpu), **glu)[:used], want) < 1e-5
