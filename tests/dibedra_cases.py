"""Small random Dibedra checkpoints, and the scenarios of the engine tests, run on the CPU (reference
ops) and on the GPU (kernels)."""
import math

import torch

import dibedra_oracle as orc
from dibedra_oracle import Oracle
from hybrid_util import feed_schedule, logits_err, make_engine, portions, random_prompts, save_checkpoint

YARN = {"factor": 3.0, "fast": 2.0, "original": 64, "slow": 0.25}


def small_config(layers="d m =1 n d", width=72, vocab=150, heads=((6, 2),), dim=20, rot=12, windows=(23, 40), ff=104, experts=7,
                 identity=2, top=3, groups=3, keep=2, eff=40, limit=1.1, scale=None, yarn=YARN, bases=(100.0, 700.0), logit_scale=0.3,
                 eps=3e-5):
    """config.json dictionary.  ``layers``: d = dense, m = experts, n = no feed-forward, =j: the weights of layer j.
    ``heads`` (query, key), ``windows`` (0: none) and ``bases`` are dealt in turn; every other rotation is stretched."""
    out = []
    for i, kind in enumerate(layers.split()):
        if kind[0] == "=":
            out.append({"weights_of": int(kind[1:])})
            continue
        H, G = heads[i % len(heads)]
        r = {"base": bases[i % len(bases)], "dims": rot, **({"scaling": dict(yarn)} if yarn and i % 2 == 0 else {})}
        mixer = {"dim": dim, "heads": H, "kv_heads": G, "rot": r, "scale": scale or 1.3 * dim ** -0.5, "vdim": dim}
        if windows[i % len(windows)]:
            mixer["mask"] = {"size": windows[i % len(windows)]}
        router = {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}, "identity": identity}
        mlp = {"d": {"ff": ff, "kind": "dense"}, "n": None,
               "m": {"expert": {"ff": eff, "limit": limit}, "kind": "moe", "router": router}}[kind]
        out.append({"mixer": mixer, "mlp": mlp, "type": "attention"})
    for la in out:
        if "weights_of" in la:
            la.update({k: v for k, v in out[la["weights_of"]].items()})
    return {"architecture": "Dibedra", "layers": out, "logit_scale": logit_scale, "norm": {"eps": eps}, "vocab": vocab,
            "width": width}


def wanted_logits(V, n, top, groups, keep, g):
    """(router logits [V, n] far from close calls, whether output 0 is to be banned): a few strong outputs, in the groups
    to be kept; outputs elsewhere that are stronger than some of them, but not than their groups' best; output 0 the
    strongest for many tokens."""
    z = torch.zeros(V, n)
    size = n // groups
    ban = size > 1 and size * keep > top
    for t in range(V):
        kept = torch.randperm(groups, generator=g)[:keep].tolist()
        inside = [o * size + e for o in kept for e in range(size) if not ban or o * size + e]
        pick = lambda o: next(e for e in torch.randperm(size, generator=g).tolist() if not ban or o * size + e)  # noqa: E731
        best = [o * size + pick(o) for o in kept]  # one in every kept group
        rest = [inside[i] for i in torch.randperm(len(inside), generator=g).tolist() if inside[i] not in best]
        for j, e in enumerate((best + rest)[:max(top, keep)]):
            z[t, e] = 4.2 - 0.35 * j if e in best else 2.4 - 0.25 * (j - len(best))
        for o in set(range(groups)) - set(kept):
            z[t, o * size + pick(o)] = 2.8 + 0.2 * float(torch.rand(1, generator=g))
    if ban:
        z[:, 0] += 2.7 * (torch.rand(V, generator=g) < 0.5)
    return z, ban


def random_weights(cfg, seed=0, sharp=2.5):
    """Random bf16 weights of a config, sized so that every mechanism matters in the logits (``sharp``: how
    peaked the attention scores are).  Some coordinates of a token's embedding name the experts it will choose, far
    from the rest, and few sublayers write there: a close call between two experts would compare rounding noise.  One
    router output is strong for many tokens and never chosen, for its correction."""
    g = torch.Generator().manual_seed(seed)
    W, V, w = cfg["width"], cfg["vocab"], {}

    def lin(name, o, i, gain=1.0):
        w[name] = torch.randn(o, i, generator=g) * gain / math.sqrt(i)

    def vec(name, n, mean, std):
        w[name] = mean + std * torch.randn(n, generator=g)

    def norm(name, alpha):
        vec(name, W, 1.2, 0.1), vec(name + ".b", W, 0.0, 0.1)
        w[name + ".alpha"] = torch.tensor(alpha)

    w["embed"] = torch.randn(V, W, generator=g)
    used = 0  # coordinates that name experts
    for i, la in enumerate(cfg["layers"]):
        if "weights_of" in la:
            continue
        p, m, mlp = f"l{i}.", la["mixer"], la["mlp"]
        H, G, D = m["heads"], m["kv_heads"], m["dim"]
        moe = mlp is not None and mlp["kind"] == "moe"
        norm(p + "norm1", 0.45)
        lin(p + "mix.q", H * D, W), lin(p + "mix.k", G * D, W, 0.9), lin(p + "mix.g", H * D, W, 2.0)
        vec(p + "mix.q.norm", D, sharp, 0.3), vec(p + "mix.k.norm", D, 1.0, 0.2)
        lin(p + "mix.o", W, H * D, 1.5)
        q = p + "mlp."
        if moe:
            ro, ff = mlp["router"], mlp["expert"]["ff"]
            E, n = ro["experts"], ro["experts"] + ro["identity"]
            for e in range(E):
                lin(f"{q}e{e}.gate", ff, W, 2.5), lin(f"{q}e{e}.up", ff, W, 2.5), lin(f"{q}e{e}.down", W, ff, 0.8)
            c = slice(used, used + n)
            used += n
            assert used <= W // 2, "a coordinate per router output"
            z, ban = wanted_logits(V, n, ro["top"], ro["groups"]["count"], ro["groups"]["keep"], g)
            corr = 0.003 * torch.randn(n, generator=g)
            corr[0] -= 1.5 * ban
            top = float(z.abs().max()) / 0.8
            w["embed"][:, c] = torch.atanh(z / top) / w[p + "norm1.alpha"]
            w[p + "norm1.b"][c] *= 0.1
            lin(q + "router", n, W, 0.15)
            w[q + "router"][:, c] += torch.diag(top / w[p + "norm1"][c])
            w[q + "correction"] = corr
        elif mlp is not None:
            lin(q + "up", mlp["ff"], W, 0.8), lin(q + "down", W, mlp["ff"])
    for k, v in w.items():
        if k.endswith(("mix.o", ".down")):
            v[:used] *= 0.1
    norm("final.norm", 0.4), lin("head", V, W, 2.0)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


def margin(cfg, w, tokens):
    """Smallest distance of a choice score (and of a group's best) from the other side of its decision."""
    worst, choose = [math.inf], orc.choose

    def watch(z, correction, count, keep, top):
        c = orc.softmax_scores(z) + correction
        b = c.view(count, -1).max(-1).values.sort(descending=True).values
        if keep < count:
            worst[0] = min(worst[0], float(b[keep - 1] - b[keep]))
        inside = torch.stack(sorted((c[i] for i in orc.best_groups(c, count, keep)), reverse=True))
        if len(inside) > top:
            worst[0] = min(worst[0], float(inside[top - 1] - inside[top]))
        return choose(z, correction, count, keep, top)

    orc.choose = watch
    try:
        Oracle(cfg, w).run(tokens)
    finally:
        orc.choose = choose
    return worst[0]


# sizes that differ from one another everywhere, sizes that coincide or are 1, one kind of layer alone, other
# orders, weights shared by several layers, windows of one token, of whole pages and none
CONFIGS = {
    "mixed": dict(),
    "shared_weights": dict(layers="m =0 d =2 =0 n =5", heads=((5, 5), (1, 1), (4, 2)), dim=10, rot=6, vocab=131, windows=(17, 1, 0),
                           experts=5, identity=1, top=2, groups=2, keep=1, logit_scale=1.0),
    "dense_only": dict(layers="d d", width=64, heads=((7, 1),), dim=34, rot=34, ff=64, vocab=128, windows=(0,),
                       yarn={**YARN, "factor": 1.0}),
    "experts_only": dict(layers="m m", width=96, experts=12, identity=0, top=1, groups=4, keep=1, eff=33, dim=16, rot=16,
                         heads=((4, 4),), windows=(16, 32)),
    "every_output": dict(layers="m d", experts=3, identity=1, top=4, groups=1, keep=1, heads=((1, 1),), dim=8, rot=2, windows=(2, 64)),
    "one_expert": dict(layers="m", experts=1, identity=0, top=1, groups=1, keep=1, width=128, eff=64, limit=40.0, windows=(48,)),
    "identity_most": dict(layers="m =0", experts=1, identity=7, top=2, groups=2, keep=2, windows=(5,), heads=((2, 2),)),
    "no_feed_forward": dict(layers="n n =0", width=200, yarn={"factor": 8.0, "fast": 32.0, "original": 40, "slow": 1.0}),
    "round_sizes": dict(layers="d m d =1", width=128, ff=192, heads=((4, 2),), dim=64, rot=32, experts=6, identity=2, top=3, groups=2,
                        keep=1, eff=64, windows=(33, 31)),
    "many_heads": dict(layers="d m", heads=((36, 2),), dim=24, rot=8, width=104, experts=11, identity=4, top=4, groups=5, keep=2),
    "long_heads": dict(layers="m d", heads=((2, 1), (3, 3)), dim=200, rot=136, windows=(30, 70), experts=4, identity=2, top=2, groups=3,
                       keep=2),
    "longest_heads": dict(layers="d =0", heads=((2, 2),), dim=328, rot=64, windows=(50,)),
}


def setup(tmp_path, name, seed=1, sharp=2.5, **over):
    cfg = small_config(**{**CONFIGS[name], **over})
    w = random_weights(cfg, seed=seed, sharp=sharp)
    return cfg, w, save_checkpoint(tmp_path / name, cfg, w)


def fast_attention(q, k, v, scale, window):
    """The oracle's attention as whole products (checked against it where it is used)."""
    T, H, _ = q.shape
    k, v = (x.repeat_interleave(H // x.shape[1], 1) for x in (k, v))
    s = torch.einsum("ihd,jhd->hij", q, k) * scale
    d = torch.arange(T)[:, None] - torch.arange(T)[None]
    s = s.masked_fill((d < 0) | (d >= (window or T)), float("-inf"))
    return torch.einsum("hij,jhd->ihd", torch.softmax(s, -1), v)


def whole_and_portions(tmp_path, device, dtype, name, tol):
    """Whole prompts, token by token, and portions of several sizes (down to two tokens, across page,
    window and tile borders) against the oracle."""
    cfg, w, path = setup(tmp_path, name, seed=len(name))
    prompts = random_prompts([1, 2, 17, 90, 149], cfg["vocab"], seed=3)
    assert min(margin(cfg, w, p) for p in prompts) > 0.015
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
    assert min(margin(cfg, w, p) for p in prompts) > 0.015
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
    """A short prompt, then hundreds of decoded tokens, past every window and the positions the stretched rotation was
    made for."""
    cfg, w, path = setup(tmp_path, "shared_weights", seed=6, sharp=3.0)
    p = random_prompts([n], cfg["vocab"], seed=5)
    assert margin(cfg, w, p[0]) > 0.015
    want = Oracle(cfg, w).logits(p[0])
    eng = make_engine(path, device, dtype, max_tokens=n + 12)
    got = feed_schedule(eng, p, [[(0, 3)]] + [[(0, 1)]] * (n - 3))[0]
    assert logits_err(got, want) < tol, logits_err(got, want)


def far_keys(tmp_path, device, dtype, tol, monkeypatch, n=900, fault=1e-2):
    """Sharp scores over a long context, whole, in portions and decoded, agree with the oracle; an attention that
    misses the first token, or the keys behind a page border far back, does not."""
    cfg, w, path = setup(tmp_path, "dense_only", seed=3, sharp=4.5, layers="n")
    p = random_prompts([n], cfg["vocab"], seed=7)
    eng = make_engine(path, device, dtype, max_tokens=n + 12)
    monkeypatch.setattr(orc, "window_attention", fast_attention)
    want = Oracle(cfg, w).logits(p[0])
    for cut in ([n], [n - 40] + [1] * 40, [333, 2, 50, 1, 16, 2]):
        got = feed_schedule(eng, p, [[(0, k)] for k in portions(n, cut)])[0]
        assert logits_err(got, want) < tol, (cut[:2], logits_err(got, want))

    def without(lo, hi):
        def attention(q, k, v, scale, window):
            out, H = fast_attention(q, k, v, scale, window), q.shape[1]
            k, v = (x.repeat_interleave(H // x.shape[1], 1) for x in (k, v))
            hide = torch.ones(len(q), len(q)).triu(1).bool()
            hide[hi:, lo:hi] = True
            s = (torch.einsum("ihd,jhd->hij", q, k) * scale).masked_fill(hide, float("-inf"))
            return torch.where(torch.arange(len(q))[:, None, None] >= hi, torch.einsum("hij,jhd->ihd", torch.softmax(s, -1), v), out)
        return attention

    for lo, hi in ((0, 1), (16, 32), (511, 513)):
        monkeypatch.setattr(orc, "window_attention", without(lo, hi))
        bad = Oracle(cfg, w).logits(p[0])
        d = (got.double().cpu() - bad)[hi:]
        assert float(((d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std()).max()) > fault, (lo, hi)


def window_edges(tmp_path, device, dtype, tol, monkeypatch, window, n=200, fault=1e-2):
    """Half of the heads ask for the last key inside the window, half for the first one outside; the comparison tells
    the window from one that is a token wider or narrower, in prompts, portions and decoding."""
    cfg = small_config(layers="n", width=64, heads=((4, 2),), dim=32, rot=32, vocab=96, windows=(window,), yarn=None, bases=(30.0,),
                       scale=32 ** -0.5)
    w = random_weights(cfg, seed=window, sharp=1.0)
    # queries (and keys) nearly alike before the rotation: a score is a function of the distance, largest at `dist`
    D = 32
    one = torch.zeros(D)
    one[::2] = 1.0
    c = torch.cat([torch.full((1, 1), 5.0), torch.zeros(1, 63)], 1)  # (reads the constant of the norm below)
    w["embed"] *= 0.5
    w["embed"][:, 0] = 4.0
    w["l0.norm1"][0], w["l0.norm1.b"][0] = 0.0, 1.0
    f = [30.0 ** (-2 * i / D) for i in range(D // 2)]
    asks = torch.zeros(4, D)
    for h, dist in enumerate((window - 1, window, window - 1, window)):
        for i, a in enumerate(f):
            asks[h, 2 * i], asks[h, 2 * i + 1] = math.cos(a * dist), -math.sin(a * dist)
    w["l0.mix.q"] = (w["l0.mix.q"] * 0.02 + asks.view(-1, 1) * c).to(torch.bfloat16)
    w["l0.mix.k"] = (w["l0.mix.k"] + (one.repeat(2)[:, None] * c)).to(torch.bfloat16)
    w["l0.mix.q.norm"] = torch.full((D,), 8.0).to(torch.bfloat16)
    w["l0.mix.k.norm"] = torch.full((D,), 1.0).to(torch.bfloat16)
    path = save_checkpoint(tmp_path / f"window{window}", cfg, w)
    p = random_prompts([n], cfg["vocab"], seed=window)
    monkeypatch.setattr(orc, "window_attention", fast_attention)
    want = Oracle(cfg, w).logits(p[0])
    eng = make_engine(path, device, dtype, max_tokens=n + 12)
    for cut in ([n], [1], [n - 60] + [1] * 60, [2], [window, 1, 2, 15, 16, 17]):
        got = feed_schedule(eng, p, [[(0, k)] for k in portions(n, cut)])[0]
        assert logits_err(got, want) < tol, (cut[:2], logits_err(got, want))
    for other in (window - 1, window + 1):
        if other:
            cfg["layers"][0]["mixer"]["mask"]["size"] = other
            bad = Oracle(cfg, w).logits(p[0])
            d = (got.double().cpu() - bad)[window + 1:]
            assert float(((d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std()).median()) > fault, other


def greedy_generation(tmp_path, device, dtype, gap, tight=False):
    """The engine's own entry point and scheduler (continuous batching, chunked and mixed prompts, one step ahead,
    graphs on the GPU, shared prefixes; ``tight``: a pool that preempts) picks the oracle's tokens.  Where the
    oracle's two best logits lie within ``gap`` of its spread either may be picked."""
    from mlopamd.runtime.sampler import SamplingParams

    cfg, w, path = setup(tmp_path, "round_sizes", seed=7)
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
            assert float(row.max() - row[t]) <= gap * float(row.std()), (len(p), t)
    if tight:
        assert eng.stats["preemptions"] > 0
    return eng
