"""Small random Regesun checkpoints, and the scenarios of the engine tests, run on the CPU (reference
ops) and on the GPU (kernels)."""
import math

import torch

from hybrid_util import feed_schedule, logits_err, make_engine, portions, random_prompts, save_checkpoint
from regesun_oracle import Oracle


def small_config(layers="madam", width=72, vocab=150, ff=104, no_ff=(), eps=3e-5, limit=1.3, max_positions=512,
                 windows=(21,), heads=3, dim=20, vdim=28, rank=44, scale=None, ssd_heads=4, ssd_vdim=12, state=20, groups=2,
                 conv=4, norm_groups=3, delta_heads=3, delta_dim=24):
    """config.json dictionary; ``layers``: m = mamba2, a = latent attention, d = general delta.  ``windows``
    are dealt to the attention layers in turn."""
    out, n_att = [], 0
    for i, c in enumerate(layers):
        if c == "a":
            mixer = {"dim": dim, "heads": heads, "kv_rank": rank, "mask": {"size": windows[n_att % len(windows)]},
                     "scale": scale or 1.3 * dim ** -0.5, "vdim": vdim}
            n_att += 1
        elif c == "m":
            mixer = {"conv": conv, "groups": groups, "heads": ssd_heads, "norm_groups": norm_groups, "state": state,
                     "vdim": ssd_vdim}
        else:
            mixer = {"dim": delta_dim, "heads": delta_heads}
        out.append({"type": {"a": "latent_attention", "m": "mamba2", "d": "general_delta"}[c], "mixer": mixer,
                    "mlp": None if i in no_ff else {"ff": ff, "kind": "dense", "limit": limit}})
    return {"architecture": "Regesun", "layers": out, "max_positions": max_positions, "norm": {"eps": eps},
            "vocab": vocab, "width": width}


def random_weights(cfg, seed=0, rank=7, sharp=2.5):
    """Random bf16 weights of a config, sized so that every mechanism matters in the logits (``sharp``:
    how peaked the attention scores are)."""
    g = torch.Generator().manual_seed(seed)
    W, w = cfg["width"], {}

    def lin(name, o, i, gain=1.0):
        w[name] = torch.randn(o, i, generator=g) * gain / math.sqrt(i)

    def vec(name, n, mean, std):
        w[name] = mean + std * torch.randn(n, generator=g)

    lin("embed", cfg["vocab"], W, math.sqrt(W)), lin("pos", cfg["max_positions"], W, 0.5 * math.sqrt(W))
    for i, la in enumerate(cfg["layers"]):
        p, m = f"l{i}.", la["mixer"]
        if la["type"] == "latent_attention":
            H, D, V, R = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
            lin(p + "mix.q", H * D, W), lin(p + "mix.dkv", R, W), vec(p + "mix.dkv.norm", R, 1.0, 0.2)
            lin(p + "mix.uk", H * D, R, sharp), lin(p + "mix.uv", H * V, R), vec(p + "mix.sink", H, 1.0, 1.5)
            lin(p + "mix.g", H * V, W), lin(p + "mix.o", W, H * V)
        elif la["type"] == "mamba2":
            H, inner = m["heads"], m["heads"] * m["vdim"]
            C = inner + 2 * m["groups"] * m["state"]
            lin(p + "mix.in", inner + C + H, W), vec(p + "mix.dt_bias", H, -1.0, 1.5), vec(p + "mix.A_log", H, -0.5, 1.5)
            lin(p + "mix.conv", C, m["conv"], 1.2), vec(p + "mix.conv.b", C, 0.0, 0.3), vec(p + "mix.D", H, 1.2, 0.2)
            vec(p + "mix.norm", inner, 1.0, 0.2), lin(p + "mix.o", W, inner)
        else:
            n = m["heads"] * m["dim"]
            for k in "rkvga":
                lin(p + f"mix.{k}", n, W)
            vec(p + "mix.a.b", n, 0.0, 1.5), lin(p + "mix.w1", rank, W), lin(p + "mix.w2", n, rank, 2.0)
            vec(p + "mix.w0", n, -2.0, 2.0), vec(p + "mix.norm", n, 1.0, 0.2), lin(p + "mix.o", W, n)
        for q in (1, 2) if la["mlp"] else (1,):
            vec(p + f"norm{q}", W, 1.0, 0.2), vec(p + f"norm{q}b", W, 1.0, 0.2), vec(p + f"ls{q}", W, 0.7, 0.3)
        if la["mlp"]:
            ff = la["mlp"]["ff"]
            lin(p + "mlp.gate", ff, W), lin(p + "mlp.up", ff, W), lin(p + "mlp.down", W, ff)
    vec("final.norm", W, 1.0, 0.2), lin("head", cfg["vocab"], W, 2.0)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


# sizes that differ from one another everywhere, sizes that coincide or are 1, one kind of layer alone,
# other layer orders, windows that differ between layers, feed-forwards in some layers only
CONFIGS = {
    "mixed": dict(),
    "delta_first": dict(layers="dmaad", no_ff=(0, 2), windows=(9, 40), groups=1, norm_groups=1, conv=3, vocab=131),
    "attention_only": dict(layers="aa", width=64, heads=7, dim=34, vdim=50, rank=70, windows=(1, 33), ff=64, vocab=128),
    "state_space_only": dict(layers="mm", ssd_heads=6, ssd_vdim=20, state=9, groups=3, conv=2, norm_groups=6, no_ff=(0, 1)),
    "delta_only": dict(layers="dd", delta_heads=1, delta_dim=64, width=128, limit=6.0),
    # every product on the package's own kernels: decode runs from captured graphs
    "native": dict(layers="amdm", width=128, ff=192, heads=4, dim=24, vdim=16, rank=64, windows=(48,), ssd_heads=4, ssd_vdim=32,
                   state=16, groups=2, norm_groups=2, delta_heads=2, delta_dim=32, vocab=150),
    "many_heads": dict(layers="ad", heads=36, dim=8, vdim=8, rank=140, windows=(60,), delta_heads=5, delta_dim=17, conv=1),
    "long_conv": dict(layers="ma", conv=7, ssd_heads=1, ssd_vdim=33, state=70, groups=1, norm_groups=1, windows=(400,), heads=1),
}


# a delta head's first output is the sign of r . k times the unit value: weights whose first tokens have
# r . k near zero would compare rounding noise
SEEDS = {"delta_first": 14, "many_heads": 12}


def setup(tmp_path, name, seed=1, sharp=2.5, **over):
    cfg = small_config(**{**CONFIGS[name], **over})
    w = random_weights(cfg, seed=seed, sharp=sharp, rank=1 + 6 * (seed % 3))
    return cfg, w, save_checkpoint(tmp_path / name, cfg, w)


def whole_and_portions(tmp_path, device, dtype, name, tol):
    """Whole prompts, token by token, and portions of several sizes (down to two tokens, across page,
    block, chunk and window borders) against the oracle."""
    cfg, w, path = setup(tmp_path, name, seed=SEEDS.get(name, len(name) + 1))
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
    slots used again (a pool that holds four live requests, nine in all)."""
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
    # every request again, alone, from reused pages and slots
    alone = feed_schedule(eng, prompts, [[(r, len(p))] for r, p in enumerate(prompts)])
    for a, o in zip(alone, got):
        assert logits_err(a, o) < tol


def long_decoding(tmp_path, device, dtype, tol, n=260):
    """A short prompt, then hundreds of decoded tokens: windows that pass over decoded tokens, states
    that forget slowly."""
    cfg, w, path = setup(tmp_path, "delta_first", seed=6, sharp=3.0, windows=(37, 120))
    for k in w:
        if k.endswith("A_log"):
            w[k] -= 3
        if k.endswith("w0"):
            w[k] -= 3
    save_checkpoint(path, cfg, w)
    p = random_prompts([n], cfg["vocab"], seed=5)
    want = Oracle(cfg, w).logits(p[0])
    eng = make_engine(path, device, dtype, max_tokens=n + 12)
    got = feed_schedule(eng, p, [[(0, 3)]] + [[(0, 1)]] * (n - 3))[0]
    assert logits_err(got, want) < tol, logits_err(got, want)


def window_edges(tmp_path, device, dtype, tol, fault=1e-2):
    """One attention layer with sharp scores: prompts, portions and decoding across the window's edge agree
    with the oracle, and would not with a window one token wider or narrower."""
    for window in (1, 2, 16, 31, 32, 33, 64, 90):
        cfg, w, path = setup(tmp_path, "attention_only", seed=3, sharp=12.0, layers="a", windows=(window,), max_positions=256)
        p = random_prompts([150], cfg["vocab"], seed=window)
        eng = make_engine(path, device, dtype, max_tokens=192)
        want = Oracle(cfg, w).logits(p[0])
        for cut in ([150], [95] + [1] * 55, [31, 2, 50, 1, 16, 2]):
            got = feed_schedule(eng, p, [[(0, n)] for n in portions(150, cut)])[0]
            assert logits_err(got, want) < tol, (window, cut[:2], logits_err(got, want))
        for off in (-1, 1):
            if window + off:
                cfg["layers"][0]["mixer"]["mask"]["size"] = window + off
                assert logits_err(got, Oracle(cfg, w).logits(p[0])) > fault, (window, off)


def greedy_generation(tmp_path, device, dtype, margin, tight=False):
    """The engine's own entry point and scheduler (continuous batching, chunked and mixed prompts, one
    step ahead, graphs on the GPU; ``tight``: a pool that preempts) picks the oracle's tokens.  Where
    the oracle's two best logits lie within ``margin`` of its spread either may be picked."""
    from mlopamd.runtime.sampler import SamplingParams

    cfg, w, path = setup(tmp_path, "native", seed=7)
    oracle = Oracle(cfg, w)
    eng = make_engine(path, device, dtype, max_tokens=256, seqs=3, max_num_batched_tokens=48, mixed_min_chunk=8,
                      max_model_len=256, num_kv_blocks=8 if tight else 40)
    assert not eng.prefix_caching  # a recurrent state is no part of the cached pages
    prompts = random_prompts([30, 62, 14, 31, 18] if tight else [5, 70, 1, 31, 18], cfg["vocab"], seed=8)
    outs = eng.generate(prompts, SamplingParams(max_tokens=10, ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert len(o) == 10
        lg = oracle.logits(p + o[:-1])[len(p) - 1:]
        for row, t in zip(lg, o):
            assert float(row.max() - row[t]) <= margin * float(row.std()), (len(p), t)
    if tight:
        assert eng.stats["preemptions"] > 0
    assert eng.alloc.num_free == eng.alloc.num_blocks - 1
    return eng
