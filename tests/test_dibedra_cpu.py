"""Dibedra on the CPU: configuration, loader, engine bookkeeping (pages, windows, shared weights, portions,
batches) on the reference ops against the plain oracle, and the trace runner."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import dibedra_cases as cases
import dibedra_oracle as orc
from dibedra_oracle import Oracle
from hybrid_util import logits_err, make_engine, random_prompts, rel_err, save_checkpoint
from mlopamd import ops
from mlopamd.models import build_model
from mlopamd.models.config import DibedraConfig, MoESpec, YarnSpec, get_config
from mlopamd.models.loader import load_pretrained
from mlopamd.runtime.sampler import SamplingParams

CPU, F32 = torch.device("cpu"), torch.float32
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
SLOW_ATTENTION = orc.window_attention


@pytest.fixture(autouse=True)
def products(monkeypatch):
    """The oracle's attention in whole products (test_fast_attention compares it with the loops)."""
    monkeypatch.setattr(orc, "window_attention", cases.fast_attention)


@pytest.mark.parametrize("window", [0, 1, 4, 19, 20, 50])
def test_fast_attention(window):
    g = torch.Generator().manual_seed(0)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)  # noqa: E731
    q, k, v = r(20, 6, 5), r(20, 2, 5), r(20, 2, 7)
    assert rel_err(cases.fast_attention(q, k, v, 0.7, window), SLOW_ATTENTION(q, k, v, 0.7, window)) < 1e-12


@pytest.mark.parametrize("name", list(cases.CONFIGS))
def test_whole_and_portions(tmp_path, name):
    cases.whole_and_portions(tmp_path, CPU, F32, name, 2e-4)


def test_batches(tmp_path):
    cases.batches(tmp_path, CPU, F32, 2e-4)


def test_long_decoding(tmp_path):
    cases.long_decoding(tmp_path, CPU, F32, 2e-4, n=140)


def test_far_keys(tmp_path, monkeypatch):
    cases.far_keys(tmp_path, CPU, F32, 2e-4, monkeypatch, n=620)


@pytest.mark.parametrize("window", [1, 2, 16, 17, 48])
def test_window_edges(tmp_path, monkeypatch, window):
    cases.window_edges(tmp_path, CPU, F32, 2e-4, monkeypatch, window, n=120)


@pytest.mark.parametrize("tight", [False, True])
def test_greedy_generation(tmp_path, tight):
    eng = cases.greedy_generation(tmp_path, CPU, F32, 1e-3, tight=tight)
    assert tight or eng.stats["prefix_hit_tokens"] >= 48


def test_gelu():
    x = torch.cat([torch.linspace(-12, 12, 301), torch.tensor([0.0, -1e-4, 1e-4, -1e-2])])
    assert rel_err(ops.gelu_tanh(x.clone()), orc.gelu_tanh(x.double())) < 1e-6


def routing_case(T, n, groups, seed):
    """Logits and corrections without ties: [T, n], [n]."""
    g = torch.Generator().manual_seed(seed)
    return 2 * torch.randn(T, n, generator=g), 0.3 * torch.randn(n, generator=g)


ROUTES = [(5, 2, 3, 1, 1), (1, 0, 1, 1, 1), (9, 0, 9, 3, 3), (12, 3, 4, 5, 2), (1, 7, 2, 2, 2), (40, 8, 6, 4, 1), (6, 6, 12, 1, 1),
          (3, 5, 2, 8, 3), (250, 6, 24, 16, 5), (63, 1, 20, 64, 40)]


@pytest.mark.parametrize("E,identity,top,groups,keep", ROUTES)
def test_moe_dispatch(E, identity, top, groups, keep):
    """Every token's rows, through ``inv``, and weights; identity experts have none."""
    n = E + identity
    z, corr = routing_case(33, n, groups, seed=E)
    x = torch.linalg.qr(torch.randn(33, 33, generator=torch.Generator().manual_seed(1)))[0]
    d = ops.moe_dispatch_groups(x, (x.T @ z).T.contiguous(), corr, E, top, groups, keep)  # row t of x has logits z[t]
    off = d.offsets.tolist()
    for t in range(33):
        want = dict(orc.choose(z[t].double(), corr.double(), groups, keep, top))
        rows = [(r, float(s)) for r, s in zip(d.inv[t].tolist(), d.top_w[t]) if r >= 0]
        got = {next(e for e in range(E) if off[e] <= r < off[e + 1]): s for r, s in rows}
        assert got.keys() == {e for e in want if e < E}
        assert all(abs(s - float(want[e])) < 1e-5 for e, s in got.items())
        assert all(torch.equal(d.x[r], x[t]) for r, _ in rows)
        own = sum(float(s) for e, s in want.items() if e >= E)
        assert identity == 0 or abs(float(d.self_w[t]) - own) < 1e-5
    assert (d.self_w is None) == (identity == 0)


def _each(w, *suffixes, fn):
    w.update({k: fn(v) for k, v in w.items() if k.endswith(suffixes)})


def _layers(c, **kw):
    [la["mixer"].update(kw) for la in c["layers"]]


def _yarn(c, **kw):
    [la["mixer"]["rot"].update(scaling={**la["mixer"]["rot"]["scaling"], **kw}) for la in c["layers"] if "scaling" in la["mixer"]["rot"]]


def _moe(c, part, **kw):
    [la["mlp"][part].update(kw) for la in c["layers"] if la["mlp"] and la["mlp"]["kind"] == "moe"]


# each mechanism left out or off by a little, in the oracle's configuration and weights: the comparison
# must see it
FAULTS = {
    "score scale": lambda c, w: _layers(c, scale=c["layers"][0]["mixer"]["scale"] * 1.1),
    "rotation base": lambda c, w: c["layers"][1]["mixer"]["rot"].update(base=1000.0),
    "stretch left out": lambda c, w: [la["mixer"]["rot"].pop("scaling", 0) for la in c["layers"]],
    "stretch factor": lambda c, w: _yarn(c, factor=3.6),
    "stretch range": lambda c, w: _yarn(c, original=200),
    "stretch, fast end": lambda c, w: _yarn(c, fast=0.9),
    "stretch, slow end": lambda c, w: _yarn(c, slow=0.06),
    "rotated dims": lambda c, w: [la["mixer"]["rot"].update(dims=10) for la in c["layers"]],
    "window a token wider": lambda c, w: c["layers"][0]["mixer"]["mask"].update(size=24),
    "window a token narrower": lambda c, w: c["layers"][1]["mixer"]["mask"].update(size=39),
    "window left out": lambda c, w: c["layers"][1]["mixer"].pop("mask"),
    "query norm weight": lambda c, w: _each(w, "q.norm", fn=lambda v: v * 0 + v.mean()),
    "key norm weight": lambda c, w: _each(w, "k.norm", fn=torch.ones_like),
    "gate left out": lambda c, w: _each(w, "mix.g", fn=lambda v: v * 0),
    "gates of another head": lambda c, w: _each(w, "mix.g", fn=lambda v: v.roll(20, 0)),
    "key heads swapped": lambda c, w: _each(w, "mix.k", fn=lambda v: v.roll(20, 0)),
    "norm's alpha": lambda c, w: _each(w, "norm1.alpha", fn=lambda v: v * 1.05),
    "norm's weight": lambda c, w: _each(w, ".norm1", fn=lambda v: v * 0 + 1.2),
    "norm's b": lambda c, w: _each(w, "norm1.b", fn=lambda v: v * 0),
    "last norm's alpha": lambda c, w: _each(w, "final.norm.alpha", fn=lambda v: v * 1.05),
    "last norm's b": lambda c, w: _each(w, "final.norm.b", fn=lambda v: v * 0),
    "eps": lambda c, w: c["norm"].update(eps=0.05),
    "logit scale": lambda c, w: c.update(logit_scale=c["logit_scale"] * 1.05),
    "weights of the wrong layer": lambda c, w: c["layers"][2].update(weights_of=0, mlp=c["layers"][0]["mlp"]),
    "fewer experts": lambda c, w: _moe(c, "router", top=2),
    "one more expert": lambda c, w: _moe(c, "router", top=4),
    "every group kept": lambda c, w: _moe(c, "router", groups={"count": 3, "keep": 3}),
    "one group kept": lambda c, w: _moe(c, "router", groups={"count": 3, "keep": 1}),
    "correction left out": lambda c, w: _each(w, "correction", fn=lambda v: v * 0),
    "experts' limit": lambda c, w: _moe(c, "expert", limit=1.3),
    "experts swapped": lambda c, w: w.update({"l1.mlp.e0.down": w["l1.mlp.e1.down"], "l1.mlp.e1.down": w["l1.mlp.e0.down"]}),
}
# mistakes in a mechanism's equations
FAULTY_FUNCTIONS = {
    "rotation of halves": ("rotate", lambda f: lambda x, rot: f(torch.cat([x[..., ::2], x[..., 1::2]], -1), rot)),
    "positions of queries from one": ("rotate", lambda f: lambda x, rot: f(x, rot, int(x.shape[1] == 6))),
    "values behind the norm": ("values_of", lambda f: lambda k: orc.rms(k, 3e-5)),
    "first token unseen": ("window_attention", lambda f: lambda q, k, v, s, w: torch.cat(
        [f(q, k, v, s, w)[:1], f(q[1:], k[1:], v[1:], s, w)])),
    "own token unseen": ("window_attention", lambda f: lambda q, k, v, s, w: torch.cat(
        [f(q[:1], k[:1], v[:1], s, w), f(q[1:], k[:-1], v[:-1], s, w and w - 1)])),
    "key heads dealt in turn": ("window_attention", lambda f: lambda q, k, v, s, w: f(
        q.view(len(q), 3, 2, -1).transpose(1, 2).flatten(1, 2), k, v, s, w).view(len(q), 2, 3, -1).transpose(1, 2).flatten(1, 2)),
    "one norm over all heads": ("head_norm", lambda f: lambda x, w, eps: orc.rms(x.flatten(1), eps).view(x.shape) * w),
    "head norm left out": ("head_norm", lambda f: lambda x, w, eps: x * w),
    "gate without the sigmoid": ("output_gate", lambda f: lambda o, z: o * z),
    "norm over the row": ("dynamic_tanh", lambda f: lambda x, a, w, b: orc.rms(x, 3e-5) * w + b),
    "exact gelu": ("gelu_tanh", lambda f: lambda z: torch.nn.functional.silu(z)),
    "gate's lower bound": ("clamped_unit", lambda f: lambda g, u, lim: f(g.clamp(min=-lim), u, lim)),
    "unbounded upper part": ("clamped_unit", lambda f: lambda g, u, lim: g.clamp(max=lim) * torch.sigmoid(1.702 * g.clamp(max=lim)) * (u + 1)),
    "unit without the one": ("clamped_unit", lambda f: lambda g, u, lim: f(g, u.clamp(-lim, lim) - 1, 1e9)),
    "slope of one": ("clamped_unit", lambda f: lambda g, u, lim: f(g, u, lim) * torch.sigmoid(g.clamp(max=lim)) / torch.sigmoid(1.702 * g.clamp(max=lim))),
    "weights renormalized": ("choose", lambda f: lambda z, *a: [(e, s / sum(v for _, v in f(z, *a))) for e, s in f(z, *a)]),
    "weights with the correction": ("choose", lambda f: lambda z, c, *a: [(e, s + 10 * c[e]) for e, s in f(z, c, *a)]),
    "scores over the chosen": ("choose", lambda f: lambda z, *a: list(zip([e for e, _ in f(z, *a)], orc.softmax_scores(
        z[[e for e, _ in f(z, *a)]])))),
    "identity left out": ("identity_expert", lambda f: lambda h: h * 0),
    "other groups at zero": ("best_groups", lambda f: lambda c, count, keep: set(range(len(c)))),
}


@pytest.fixture(scope="module")
def mixed_run(tmp_path_factory):
    cfg, w, path = cases.setup(tmp_path_factory.mktemp("mixed"), "mixed", seed=11, sharp=3.0)
    p = random_prompts([70], cfg["vocab"], seed=2)[0]
    eng = make_engine(path, CPU, F32, max_tokens=80)
    got = eng.feed([(eng.open_sequence(), p, list(range(70)))])
    assert logits_err(got, Oracle(cfg, w).logits(p)) < 2e-4
    return cfg, w, p, got


@pytest.mark.parametrize("fault", [*FAULTS, *FAULTY_FUNCTIONS])
def test_comparison_sees_faults(mixed_run, monkeypatch, fault):
    cfg, w, p, got = mixed_run
    cfg, w = json.loads(json.dumps(cfg)), {k: v.double() for k, v in w.items()}
    if fault in FAULTS:
        FAULTS[fault](cfg, w)
    else:
        name, wrap = FAULTY_FUNCTIONS[fault]
        monkeypatch.setattr(orc, name, wrap(getattr(orc, name)))
    assert logits_err(got, Oracle(cfg, w).logits(p)) > 5e-3, fault


def test_loader_builds_the_configured_model(tmp_path):
    cfg, w, path = cases.setup(tmp_path, "shared_weights", seed=2)
    m = load_pretrained(path, device="cpu", dtype=F32)
    c = m.cfg
    assert isinstance(c, DibedraConfig) and len(c.layers) == 7
    assert [(la.mixer.heads, la.mixer.kv_heads) for la in c.layers] == [(5, 5), (5, 5), (4, 2), (4, 2), (5, 5), (4, 2), (4, 2)]
    assert [la.weights_of for la in c.layers] == [-1, 0, -1, 2, 0, -1, 5]
    assert [la.mixer.window for la in c.layers] == [17, 17, 0, 0, 17, 0, 0]
    assert [la.mixer.scaling is not None for la in c.layers] == [True, True, True, True, True, False, False]
    assert c.layers[0].mixer.scaling == YarnSpec(3.0, 64.0, 2.0, 0.25)
    assert c.layers[0].moe == MoESpec(5, 2, 40, scores="softmax", identity=1, groups=2, keep=1, correction=True, limit=1.1)
    assert c.layers[2].ff == 104 and c.layers[5].ff == 0 and not c.layers[5].moe
    assert c.rms_eps == cfg["norm"]["eps"] and c.logit_scale == 1.0
    assert c.num_params() == sum(v.numel() for v in w.values())
    # weights are shared, pages are not
    assert m.layers[0] is m.layers[1] is m.layers[4] and m.layers[2] is m.layers[3] and len(m.weights) == 3
    assert [(la.n_kv, la.k_dim, la.v_dim) for la in m.cache_layout] == [(5, 64, 64)] * 2 + [(2, 64, 64)] * 2 + [(5, 64, 64)] + [(2, 64, 64)] * 2
    assert c.kv_bytes_per_token() == 2 * 2 * 10 * (3 * 5 + 4 * 2) and not m.state_shapes
    assert c.eos_ids == (-1,) and 0 < c.active_params() and 0 < c.flops_per_token()


def test_weights_of_a_later_layer_and_of_a_sharing_one(tmp_path):
    """Shared weights by way of a layer that shares them itself, or that comes later."""
    cfg, w, _ = cases.setup(tmp_path, "shared_weights", seed=2)
    p = random_prompts([30], cfg["vocab"], seed=1)[0]
    want = Oracle(cfg, w).logits(p)
    cfg["layers"][4]["weights_of"] = 1
    turned = json.loads(json.dumps(cfg))
    turned["layers"][0]["weights_of"] = 4
    del turned["layers"][4]["weights_of"]
    turned["layers"][1]["weights_of"] = 0
    for c, ww in ((cfg, w), (turned, {k.replace("l0.", "l4."): v for k, v in w.items()})):
        eng = make_engine(save_checkpoint(tmp_path / f"x{len(ww)}{id(c)}", c, ww), CPU, F32, max_tokens=64)
        got = eng.feed([(eng.open_sequence(), p, list(range(30)))])
        assert logits_err(got, want) < 2e-4


@pytest.mark.parametrize("change", [lambda d: d["layers"][0].update(type="latent_attention"), lambda d: d.update(extra=1),
                                    lambda d: d["layers"][0]["mixer"].update(sink=True),
                                    lambda d: d["layers"][0]["mixer"].update(vdim=16),
                                    lambda d: d["layers"][0]["mixer"].update(kv_heads=4),
                                    lambda d: d["layers"][0]["mixer"]["mask"].update(kind="chunk"),
                                    lambda d: d["layers"][0]["mixer"]["rot"].update(style="halves"),
                                    lambda d: d["layers"][0]["mixer"]["rot"].update(dims=22),
                                    lambda d: d["layers"][0]["mixer"]["rot"]["scaling"].update(kind="linear"),
                                    lambda d: d["layers"][2].update(weights_of=2),
                                    lambda d: d["layers"][2].update(weights_of=5),
                                    lambda d: d["layers"][2].update(weights_of=0),
                                    lambda d: d["layers"][2].update(mlp=None),
                                    lambda d: d["layers"][1]["mlp"].update(shared={"ff": 8}),
                                    lambda d: d["layers"][1]["mlp"]["router"].update(scores="sigmoid"),
                                    lambda d: d["layers"][1]["mlp"]["router"].update(top=7),
                                    lambda d: d["layers"][1]["mlp"]["router"]["groups"].update(count=2),
                                    lambda d: d["layers"][1]["mlp"]["router"]["groups"].update(keep=4),
                                    lambda d: d["layers"][1]["mlp"]["expert"].update(limit=0),
                                    lambda d: d["layers"][1]["mlp"].update(kind="switch"),
                                    lambda d: d["layers"][0]["mlp"].update(bias=True),
                                    lambda d: d["norm"].update(kind="layer"),
                                    lambda d: d.update(architecture="Other")])
def test_loader_refuses_what_it_does_not_know(tmp_path, change):
    cfg = cases.small_config()
    save_checkpoint(tmp_path, cfg, cases.random_weights(cfg))
    load_pretrained(tmp_path, device="cpu", dtype=F32)
    change(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    with pytest.raises((ValueError, KeyError)):
        load_pretrained(tmp_path, device="cpu", dtype=F32)


def test_wrong_tensor_shape_is_refused(tmp_path):
    cfg = cases.small_config()
    w = cases.random_weights(cfg)
    w["l1.mlp.e2.down"] = w["l1.mlp.e2.down"][:-1]
    save_checkpoint(tmp_path, cfg, w)
    with pytest.raises(ValueError, match="l1.mlp.e2.down"):
        load_pretrained(tmp_path, device="cpu", dtype=F32)


def test_absent_settings(tmp_path):
    """No mask, no groups, no identity experts, no scale: the same as their neutral values."""
    cfg, w, path = cases.setup(tmp_path, "mixed", seed=2, windows=(0,), groups=1, keep=1, identity=0, experts=9, logit_scale=1.0)
    p = random_prompts([20], cfg["vocab"], seed=1)[0]
    want = Oracle(cfg, w).logits(p)
    for la in cfg["layers"]:
        la["mixer"]["mask"] = None
        if la["mlp"] and la["mlp"]["kind"] == "moe":
            la["mlp"]["router"] = {"experts": 9, "top": 3}
    del cfg["logit_scale"]
    eng = make_engine(save_checkpoint(tmp_path / "absent", cfg, w), CPU, F32, max_tokens=64)
    assert logits_err(eng.feed([(eng.open_sequence(), p, list(range(20)))]), want) < 2e-4


def test_shared_prefixes_reuse_pages(tmp_path):
    """A prompt that begins like a finished one reads its pages, also in the layers that share weights, and generates
    what it does alone."""
    cfg, w, path = cases.setup(tmp_path, "shared_weights", seed=3)
    a, b = random_prompts([64, 20], cfg["vocab"], seed=5)
    params = SamplingParams(max_tokens=5, ignore_eos=True)
    kw = dict(max_tokens=256, max_num_batched_tokens=64)
    alone = make_engine(path, CPU, F32, **kw).generate([a[:48] + b], params)
    eng = make_engine(path, CPU, F32, **kw)
    eng.generate([a], params)
    before = eng.stats["prefill_tokens"]
    assert eng.generate([a[:48] + b], params) == alone
    assert eng.stats["prefill_tokens"] - before == 20


def test_presets_build_and_serve():
    from mlopamd.controller.placement import plan
    from mlopamd.runtime.deploy import build_engine

    cfg = get_config("dibedra-8b")
    assert 3e9 < cfg.num_params() < 10e9 and plan("dibedra-8b").tensorParallel == 1
    assert len(get_config("dibedra-8b", num_layers=6).layers) == 6
    assert plan("tiny-dibedra").fits
    eng = build_engine("tiny-dibedra", device="cpu", dtype=F32, max_num_seqs=2, max_model_len=64,
                       max_num_batched_tokens=64, num_kv_blocks=16)
    params = SamplingParams(max_tokens=6, temperature=0.8, top_k=20, seed=5, ignore_eos=True)
    out, again = eng.generate([[3, 4, 5]], params), eng.generate([[3, 4, 5]], params)
    assert len(out[0]) == 6 and out == again


def test_trace_runner_program(tmp_path):
    """bin/trace_run end to end: steps on standard input, logits files, requests that end and return."""
    cfg, w, path = cases.setup(tmp_path, "shared_weights", seed=4)
    a, b = random_prompts([23, 9], cfg["vocab"], seed=6)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:7], "want": [6, 2]}, {"id": "a", "tokens": a[20:21], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[21:], "want": [0, 1]}, {"id": "b", "tokens": b[7:], "want": [1]}], "end": ["a", "b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": b, "want": [8]}], "end": ["a"]}]
    out = tmp_path / "out"
    out.mkdir()
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(path), "--dtype", "float32", "--out",
                        str(out), "--max-tokens", "64", "--device", "cpu"],
                       input="\n".join(map(json.dumps, steps)), capture_output=True, text=True, timeout=120,
                       env={**os.environ, "PATH": os.path.dirname(sys.executable) + ":" + os.environ["PATH"]})
    assert r.returncode == 0, r.stderr
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(4)]
    assert not (out / "0.f32").exists()
    o = Oracle(cfg, w)
    la, lb = o.logits(a), o.logits(b)
    for step, want in ((1, [lb[6], lb[2], la[20]]), (2, [la[21], la[22], lb[8]]), (3, [lb[8]])):
        got = np.fromfile(out / f"{step}.f32", "<f4").reshape(len(want), cfg["vocab"])
        assert logits_err(torch.from_numpy(got), torch.stack(want)) < 2e-4


def test_tensor_parallel_is_refused():
    from mlopamd.parallel.comm import single

    ps = single()
    ps.tp.size = 2
    try:
        with pytest.raises(ValueError, match="one GPU"):
            build_model("tiny-dibedra", device="cpu", dtype=F32, pstate=ps)
    finally:
        ps.tp.size = 1
