"""Small random Nafazen checkpoints, and the scenarios of the engine tests, run on the CPU (reference
ops) and on the GPU (kernels)."""
import math

import torch

import nafazen_oracle as orc
from hybrid_util import feed_schedule, logits_err, make_engine, portions, random_prompts, save_checkpoint
from nafazen_oracle import Oracle

YARN = {"factor": 3.0, "fast": 2.0, "original": 64, "slow": 0.25}


def small_config(layers="yd pm yd sm", width=72, vocab=150, heads=(3,), dim=20, rot=12, vdim=28, rank=44, q_rank=36, ff=104,
                 experts=5, top=2, eff=40, shared=56, scale=None, yarn=YARN, bases=(100.0, 700.0), cap=11.0, embed=3.7,
                 eps=3e-5):
    """config.json dictionary.  ``layers``: two letters each; y = stretched positions, p = plain ones, s = on the
    latents of the last plain layer; d = dense, m = experts, n = no feed-forward.  ``heads`` are dealt in turn."""
    out, owner = [], None
    for i, (a, f) in enumerate(layers.split()):
        r = {"base": bases[0] if a == "y" else bases[1], "dims": rot, **({"scaling": dict(yarn)} if a == "y" else {})}
        mixer = {"dim": dim, "heads": heads[i % len(heads)], "kv_rank": rank, "q_rank": q_rank, "rot": r, "rot_dim": rot,
                 "scale": scale or 1.3 * (dim + rot) ** -0.5, "vdim": vdim}
        if a == "p":
            owner = i
        elif a == "s":
            mixer["kv_from"] = owner
        mlp = {"d": {"ff": ff, "kind": "dense"}, "n": None,
               "m": {"expert": {"ff": eff}, "kind": "moe", "router": {"experts": experts, "top": top}, "shared": {"ff": shared}}}[f]
        out.append({"mixer": mixer, "mlp": mlp, "type": "latent_attention" + ("" if a == "y" else "_2")})
    return {"architecture": "Nafazen", "embedding": {"scale": embed}, "layers": out, "logit_softcap": cap, "norm": {"eps": eps},
            "vocab": vocab, "width": width}


def random_weights(cfg, seed=0, sharp=2.5):
    """Random bf16 weights of a config, sized so that every mechanism matters in the logits (``sharp``: how
    peaked the attention scores are).  Every token's embedding names the experts it will choose, far from the
    rest: a close call between two experts would compare rounding noise."""
    g = torch.Generator().manual_seed(seed)
    W, V, w = cfg["width"], cfg["vocab"], {}

    def lin(name, o, i, gain=1.0):
        w[name] = torch.randn(o, i, generator=g) * gain / math.sqrt(i)

    def vec(name, n, mean, std):
        w[name] = mean + std * torch.randn(n, generator=g)

    def one(name, mean, std):
        w[name] = mean + std * torch.randn((), generator=g)

    lin("embed", V, W, math.sqrt(W))
    axes = torch.linalg.qr(torch.randn(W, W, generator=g))[0].T
    used = 0
    for i, la in enumerate(cfg["layers"]):
        p, m = f"l{i}.", la["mixer"]
        H, D, Vd, R, Q, r = m["heads"], m["dim"], m["vdim"], m["kv_rank"], m["q_rank"], m["rot_dim"]
        lin(p + "mix.dq", Q, W), vec(p + "mix.dq.norm", Q, 1.0, 0.2), lin(p + "mix.uq", H * (D + r), Q)
        if "kv_from" not in m:
            lin(p + "mix.dkv", R + r, W, 0.3), vec(p + "mix.dkv.norm", R, 1.0, 0.2)
        lin(p + "mix.uk", H * D, R, sharp), lin(p + "mix.uv", H * Vd, R), lin(p + "mix.o", W, H * Vd)
        one(p + "norm1", 0.8, 0.1)
        if not la["mlp"]:
            continue
        one(p + "norm2", 0.9, 0.1)
        q = p + "mlp."
        if la["mlp"]["kind"] == "dense":
            lin(q + "up", la["mlp"]["ff"], W, 0.4), lin(q + "down", W, la["mlp"]["ff"]), vec(q + "act", 2, 0.3, 0.8)
            continue
        E, top, ff, sh = (la["mlp"][a][b] for a, b in (("router", "experts"), ("router", "top"), ("expert", "ff"), ("shared", "ff")))
        for e in range(E):
            lin(f"{q}e{e}.gate", ff, W, 0.4), lin(f"{q}e{e}.up", ff, W, 0.4), lin(f"{q}e{e}.down", W, ff)
        lin(q + "shared.gate", sh, W, 0.4), lin(q + "shared.up", sh, W, 0.4), lin(q + "shared.down", W, sh, 0.6)
        lin(q + "shared.sg", 1, W, 0.4)
        u = axes[used:used + E]
        used += E
        assert used <= W, "one axis per expert"
        chosen = torch.argsort(torch.rand(V, E, generator=g), 1)[:, :top]
        level = 16 + 8 * torch.rand(V, top, generator=g)
        w["embed"] += (level[:, :, None] * u[chosen]).sum(1)
        w[q + "router"] = 0.06 * u
    w["embed"] /= cfg["embedding"]["scale"]
    one("final.norm", 1.0, 0.1), lin("head", V, W, 2.0)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


# sizes that differ from one another everywhere, sizes that coincide or are 1, one kind of layer alone, other
# orders, latents shared by several layers with other head counts, layers without a feed-forward
CONFIGS = {
    "mixed": dict(),
    "shared_latents": dict(layers="pm sd yn sm pn sd", heads=(3, 5, 2), dim=10, vdim=33, q_rank=21, rank=70, rot=6, vocab=131),
    "dense_only": dict(layers="yd pd", width=64, heads=(7,), dim=34, vdim=50, rank=64, rot=22, q_rank=64, ff=64, vocab=128,
                       yarn={**YARN, "factor": 1.0}),
    "experts_only": dict(layers="pm ym", width=96, experts=9, top=1, eff=33, shared=16, dim=16, rot=32, vdim=16, heads=(4,)),
    "every_expert": dict(layers="ym pm", experts=4, top=4, heads=(1,), dim=8, rot=2, vdim=8, rank=8, q_rank=8),
    "one_expert": dict(layers="pm", experts=1, top=1, width=128, eff=64, shared=64, cap=40.0, embed=1.0),
    "no_feed_forward": dict(layers="yn pn sn", width=200, yarn={"factor": 8.0, "fast": 32.0, "original": 40, "slow": 1.0}),
    "native": dict(layers="pm yd sm", width=128, ff=192, heads=(4,), dim=24, rot=8, vdim=16, rank=56, q_rank=64, experts=6, top=3,
                   eff=64, shared=128),
    "many_heads": dict(layers="yd pm", heads=(36,), dim=8, rot=8, vdim=8, rank=140, q_rank=100, experts=20, top=6),
}


def setup(tmp_path, name, seed=1, sharp=2.5, **over):
    cfg = small_config(**{**CONFIGS[name], **over})
    w = random_weights(cfg, seed=seed, sharp=sharp)
    return cfg, w, save_checkpoint(tmp_path / name, cfg, w)


def fast_attention(q, k, v, q_rot, k_rot, scale):
    """The oracle's attention as whole products (checked against it where it is used)."""
    s = (torch.einsum("ihd,jhd->hij", q, k) + torch.einsum("ihd,jd->hij", q_rot, k_rot)) * scale
    s = s.masked_fill(torch.ones(len(q), len(q)).triu(1).bool(), float("-inf"))
    return torch.einsum("hij,jhd->ihd", torch.softmax(s, -1), v)


def whole_and_portions(tmp_path, device, dtype, name, tol):
    """Whole prompts, token by token, and portions of several sizes (down to two tokens, across page
    and tile borders) against the oracle."""
    cfg, w, path = setup(tmp_path, name, seed=len(name))
    prompts = random_prompts([1, 2, 17, 90, 149], cfg["vocab"], seed=3)
    want = [Oracle(cfg, w).logits(p) for p in prompts]
    eng = make_engine(path, device, dtype, max_tokens=192)
    free = eng.alloc.num_free
    cuts = {"whole": [[999]] * 5, "tokens": [[1]] * 5, "twos": [[2]] * 5,
            "uneven": [[1], [2], [3, 14], [16, 1, 5, 40], [65, 2, 1, 31, 17]],
            "prompt_then_decode": [[1], [1], [12, 1], [64] + [1] * 26, [129] + [1] * 20]}
    for kind, sizes in cuts.items():
        sched = [[(r, n)] for r, p in enumerate(prompts) for n in portions(len(p), sizes[r])]
        got = feed_schedule(eng, prompts, sched)
        for a, o in zip(got, want):
            assert logits_err(a, o) < tol, (kind, len(o), logits_err(a, o))
    assert eng.alloc.num_free == free and len(eng.free_rows) == 4


def batches(tmp_path, device, dtype, tol):
    """Unequal requests in one batch, portions beside decoded tokens, requests that pause, pages and
    rows used again (a pool that holds four live requests, nine in all)."""
    cfg, w, path = setup(tmp_path, "mixed", seed=5, sharp=3.0)
    prompts = random_prompts([33, 61, 5, 100, 1, 48, 16, 77, 2], cfg["vocab"], seed=4)
    want = [Oracle(cfg, w).logits(p) for p in prompts]
    g = torch.Generator().manual_seed(9)
    left = {r: len(p) for r, p in enumerate(prompts)}
    waiting, live, sched = list(left), [], []
    while waiting or live:
        while waiting and len(live) < 4:
            live.append(waiting.pop(0))
        step = []
        for r in live:
            if len(live) > 1 and torch.rand(1, generator=g) < 0.25:
                continue  # left out of this step
            n = min(left[r], int([1, 1, 2, 7, 16, 30][torch.randint(0, 6, (1,), generator=g)]))
            left[r] -= n
            step.append((r, n))
        if step:
            sched.append(step)
        live = [r for r in live if left[r]]
    eng = make_engine(path, device, dtype, max_tokens=320)
    got = feed_schedule(eng, prompts, sched)
    for r, (a, o) in enumerate(zip(got, want)):
        assert logits_err(a, o) < tol, (r, len(o), logits_err(a, o))
    # every request again, alone, from reused pages and rows
    alone = feed_schedule(eng, prompts, [[(r, len(p))] for r, p in enumerate(prompts)])
    for a, o in zip(alone, got):
        assert logits_err(a, o) < tol


def long_decoding(tmp_path, device, dtype, tol, n=260):
    """A short prompt, then hundreds of decoded tokens, past the positions the stretched rotation was made for."""
    cfg, w, path = setup(tmp_path, "shared_latents", seed=6, sharp=3.0)
    p = random_prompts([n], cfg["vocab"], seed=5)
    want = Oracle(cfg, w).logits(p[0])
    eng = make_engine(path, device, dtype, max_tokens=n + 12)
    got = feed_schedule(eng, p, [[(0, 3)]] + [[(0, 1)]] * (n - 3))[0]
    assert logits_err(got, want) < tol, logits_err(got, want)


def far_keys(tmp_path, device, dtype, tol, monkeypatch, n=900, fault=1e-2):
    """Sharp scores over a long context, whole, in portions and decoded, agree with the oracle; an attention that
    misses the first token, or the keys behind a page border far back, does not."""
    cfg, w, path = setup(tmp_path, "dense_only", seed=3, sharp=5.0, layers="pn")
    p = random_prompts([n], cfg["vocab"], seed=7)
    eng = make_engine(path, device, dtype, max_tokens=n + 12)
    monkeypatch.setattr(orc, "causal_attention", fast_attention)
    want = Oracle(cfg, w).logits(p[0])
    for cut in ([n], [n - 40] + [1] * 40, [333, 2, 50, 1, 16, 2]):
        got = feed_schedule(eng, p, [[(0, k)] for k in portions(n, cut)])[0]
        assert logits_err(got, want) < tol, (cut[:2], logits_err(got, want))

    def without(lo, hi):
        def attention(q, k, v, q_rot, k_rot, scale):
            k_rot, k, far = k_rot.clone(), k.clone(), torch.zeros(len(q), 1, 1, dtype=q.dtype)
            out = fast_attention(q, k, v, q_rot, k_rot, scale)
            s = (torch.einsum("ihd,jhd->hij", q, k) + torch.einsum("ihd,jd->hij", q_rot, k_rot)) * scale
            hide = torch.ones(len(q), len(q)).triu(1).bool()
            hide[hi:, lo:hi] = True
            return far + torch.where(torch.arange(len(q))[:, None, None] >= hi,
                                     torch.einsum("hij,jhd->ihd", torch.softmax(s.masked_fill(hide, float("-inf")), -1), v), out)
        return attention

    for lo, hi in ((0, 1), (16, 32), (511, 513)):
        monkeypatch.setattr(orc, "causal_attention", without(lo, hi))
        bad = Oracle(cfg, w).logits(p[0])
        d = (got.double().cpu() - bad)[hi:]
        assert float(((d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std()).max()) > fault, (lo, hi)


def greedy_generation(tmp_path, device, dtype, margin, tight=False):
    """The engine's own entry point and scheduler (continuous batching, chunked and mixed prompts, one step ahead,
    graphs on the GPU, shared prefixes; ``tight``: a pool that preempts) picks the oracle's tokens.  Where the
    oracle's two best logits lie within ``margin`` of its spread either may be picked."""
    from mlopamd.runtime.sampler import SamplingParams

    cfg, w, path = setup(tmp_path, "native", seed=7)
    oracle = Oracle(cfg, w)
    eng = make_engine(path, device, dtype, max_tokens=256, seqs=3, max_num_batched_tokens=48, mixed_min_chunk=8,
                      max_model_len=256, num_kv_blocks=8 if tight else 40)
    assert eng.prefix_caching  # a sequence's pages are all of its state
    prompts = random_prompts([30, 62, 14, 31, 18] if tight else [5, 70, 1, 31, 18], cfg["vocab"], seed=8)
    if not tight:
        prompts.append(prompts[1][:50] + prompts[3])  # begins like another
    outs = eng.generate(prompts, SamplingParams(max_tokens=10, ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert len(o) == 10
        lg = oracle.logits(p + o[:-1])[len(p) - 1:]
        for row, t in zip(lg, o):
            assert float(row.max() - row[t]) <= margin * float(row.std()), (len(p), t)
    if tight:
        assert eng.stats["preemptions"] > 0
    return eng
