"""Nafazen on the CPU: configuration, loader, engine bookkeeping (pages, shared latents, portions,
batches) on the reference ops against the plain oracle, and the trace runner."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import nafazen_cases as cases
import nafazen_oracle as orc
from hybrid_util import logits_err, make_engine, random_prompts, rel_err, save_checkpoint
from mlopamd import ops
from mlopamd.models import build_model
from mlopamd.models.config import MoESpec, NafazenConfig, RotarySpec, YarnSpec, get_config
from mlopamd.models.layers import rotary_table
from mlopamd.models.loader import load_pretrained
from mlopamd.runtime.sampler import SamplingParams
from nafazen_oracle import Oracle

CPU, F32 = torch.device("cpu"), torch.float32
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.fixture(autouse=True)
def products(monkeypatch):
    """The oracle's attention in whole products (test_fast_attention compares it with the loops)."""
    monkeypatch.setattr(orc, "causal_attention", cases.fast_attention)


SLOW_ATTENTION = orc.causal_attention


def test_fast_attention():
    g = torch.Generator().manual_seed(0)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)  # noqa: E731
    q, k, v, qr, kr = r(19, 3, 5), r(19, 3, 5), r(19, 3, 7), r(19, 3, 4), r(19, 4)
    assert rel_err(cases.fast_attention(q, k, v, qr, kr, 0.7), SLOW_ATTENTION(q, k, v, qr, kr, 0.7)) < 1e-12


@pytest.mark.parametrize("name", list(cases.CONFIGS))
def test_whole_and_portions(tmp_path, name):
    cases.whole_and_portions(tmp_path, CPU, F32, name, 2e-4)


def test_batches(tmp_path):
    cases.batches(tmp_path, CPU, F32, 2e-4)


def test_long_decoding(tmp_path):
    cases.long_decoding(tmp_path, CPU, F32, 2e-4, n=140)


def test_far_keys(tmp_path, monkeypatch):
    cases.far_keys(tmp_path, CPU, F32, 2e-4, monkeypatch, n=620)


@pytest.mark.parametrize("tight", [False, True])
def test_greedy_generation(tmp_path, tight):
    eng = cases.greedy_generation(tmp_path, CPU, F32, 1e-3, tight=tight)
    assert tight or eng.stats["prefix_hit_tokens"] >= 48


@pytest.mark.parametrize("dims,base,yarn", [(12, 100.0, cases.YARN), (64, 5e5, {"factor": 4.0, "fast": 32.0, "original": 4096, "slow": 1.0}),
                                            (2, 50.0, {"factor": 2.0, "fast": 1.0, "original": 30, "slow": 1.0}),
                                            (32, 1e4, {"factor": 16.0, "fast": 1e9, "original": 512, "slow": 1e-9}), (8, 300.0, None)])
def test_rotary_table(dims, base, yarn):
    """Against the oracle's rotation of unit vectors; ramps that are empty, whole, or cut at the ends."""
    spec = RotarySpec(base, dims, yarn and YarnSpec(yarn["factor"], yarn["original"], yarn["fast"], yarn["slow"]))
    t = rotary_table(spec, 300)
    x = torch.zeros(300, 1, dims, dtype=torch.float64)
    x[:, 0, ::2] = 1
    want = orc.rotate(x, {"base": base, "dims": dims, **({"scaling": yarn} if yarn else {})})[:, 0]
    assert rel_err(t[:, :dims // 2], want[:, ::2]) < 1e-6 and rel_err(t[:, dims // 2:], want[:, 1::2]) < 1e-6


def test_xielu():
    x = torch.cat([torch.linspace(-9, 9, 201), torch.tensor([0.0, -1e-4, 1e-4, -1e-2])])
    for p, q in ((0.3, -1.1), (-2.0, 1.5), (0.0, 0.0)):
        a, b = orc.softplus(torch.tensor(p)).item(), 0.5 + orc.softplus(torch.tensor(q)).item()
        want = orc.xielu(x.double(), torch.tensor(p, dtype=torch.float64), torch.tensor(q, dtype=torch.float64))
        assert rel_err(ops.xielu(x.clone(), a, b), want) < 1e-6


@pytest.mark.parametrize("E,top,gated", [(5, 2, True), (1, 1, False), (9, 9, True), (40, 3, False)])
def test_moe_dispatch(E, top, gated):
    """Every token's rows, through ``inv``: the token times the score of each expert it chose."""
    g = torch.Generator().manual_seed(E)
    x, w = torch.randn(33, 24, generator=g), torch.randn(E + gated, 24, generator=g)
    d = ops.moe_dispatch_input(x, w, E, top)
    z = x.double() @ w.double().T
    off = d.offsets.tolist()
    for t in range(33):
        got = {next(e for e in range(E) if off[e] <= r < off[e + 1]): d.x[r] for r in d.inv[t].tolist()}
        want = dict(orc.choose(z[t, :E], top))
        assert got.keys() == want.keys()
        for e, s in want.items():
            assert rel_err(got[e], s * x[t].double()) < 1e-5
    assert (d.gate is not None) == gated
    if gated:
        assert rel_err(d.gate, torch.sigmoid(z[:, E])) < 1e-6


def _each(w, *suffixes, fn):
    w.update({k: fn(v) for k, v in w.items() if k.endswith(suffixes)})


def _mixers(c, yarn=None):
    return [la["mixer"] for la in c["layers"] if yarn is None or ("scaling" in la["mixer"]["rot"]) == yarn]


def _yarn(c, **kw):
    [m["rot"].update(scaling={**m["rot"]["scaling"], **kw}) for m in _mixers(c, True)]


# each mechanism left out or off by a little, in the oracle's configuration and weights: the comparison
# must see it
FAULTS = {
    "score scale": lambda c, w: [m.update(scale=m["scale"] * 1.1) for m in _mixers(c)],
    "rotation base": lambda c, w: [m["rot"].update(base=m["rot"]["base"] * 1.5) for m in _mixers(c, False)],
    "stretch left out": lambda c, w: [m["rot"].pop("scaling") for m in _mixers(c, True)],
    "stretch factor": lambda c, w: _yarn(c, factor=3.6),
    "stretch range": lambda c, w: _yarn(c, original=200),
    "stretch, fast end": lambda c, w: _yarn(c, fast=0.9),
    "stretch, slow end": lambda c, w: _yarn(c, slow=0.06),
    "stretch on plain layers": lambda c, w: [m["rot"].update(scaling=dict(cases.YARN)) for m in _mixers(c, False)],
    "latent norm weight": lambda c, w: _each(w, "dkv.norm", fn=torch.ones_like),
    "query norm weight": lambda c, w: _each(w, "dq.norm", fn=torch.ones_like),
    "latents of another layer": lambda c, w: c["layers"][3]["mixer"].update(kv_from=2),
    "heads of the values swapped": lambda c, w: w.update({"l1.mix.uv": w["l1.mix.uv"].flip(0)}),
    "norm behind left out": lambda c, w: _each(w, ".norm1", fn=torch.ones_like),
    "second norm": lambda c, w: _each(w, ".norm2", fn=torch.ones_like),
    "last norm": lambda c, w: _each(w, "final.norm", fn=lambda v: v * 1.05),
    "norm eps": lambda c, w: c["norm"].update(eps=0.05),
    "embedding scale": lambda c, w: c["embedding"].update(scale=c["embedding"]["scale"] * 1.05),
    "logit cap": lambda c, w: c.update(logit_softcap=c["logit_softcap"] * 1.1),
    "activation's upper number": lambda c, w: _each(w, "mlp.act", fn=lambda v: v + torch.tensor([0.3, 0.0])),
    "activation's lower number": lambda c, w: _each(w, "mlp.act", fn=lambda v: v + torch.tensor([0.0, 0.3])),
    "fewer experts": lambda c, w: [la["mlp"]["router"].update(top=1) for la in c["layers"] if la["mlp"]["kind"] == "moe"],
    "one more expert": lambda c, w: [la["mlp"]["router"].update(top=3) for la in c["layers"] if la["mlp"]["kind"] == "moe"],
    "shared gate left out": lambda c, w: _each(w, "shared.sg", fn=lambda v: v * 0),
    "shared expert left out": lambda c, w: _each(w, "shared.down", fn=lambda v: v * 0),
    "experts swapped": lambda c, w: w.update({"l1.mlp.e0.down": w["l1.mlp.e1.down"], "l1.mlp.e1.down": w["l1.mlp.e0.down"]}),
}
# mistakes in a mechanism's equations
FAULTY_FUNCTIONS = {
    "rotation of halves": ("rotate", lambda f: lambda x, rot: f(torch.cat([x[..., ::2], x[..., 1::2]], -1), rot)),
    "positions from one": ("rotate", lambda f: lambda x, rot: f(x[:, :, :], rot, 1) if x.shape[1] > 1 else f(x, rot)),
    "rotated score left out": ("causal_attention", lambda f: lambda q, k, v, qr, kr, s: f(q, k, v, qr * 0, kr, s)),
    "first token unseen": ("causal_attention", lambda f: lambda q, k, v, qr, kr, s: torch.cat(
        [f(q, k, v, qr, kr, s)[:1], f(q[1:], k[1:], v[1:], qr[1:], kr[1:], s)])),
    "own token unseen": ("causal_attention", lambda f: lambda q, k, v, qr, kr, s: torch.cat(
        [v[:1], torch.stack([f(torch.cat([q[:i], q[i:i + 1]])[1:], k[:i], v[:i], qr[1:i + 1], kr[:i], s)[-1] for i in range(1, len(q))])])),
    "norm with the square root's eps outside": ("rms", lambda f: lambda x, eps: x / (torch.sqrt((x * x).mean(-1, keepdim=True)) + 0.05)),
    "weights renormalized": ("choose", lambda f: lambda z, top: [(e, s / sum(v for _, v in f(z, top))) for e, s in f(z, top)]),
    "weight on the output": ("weighted_expert", lambda f: lambda ff, h, w: w * ff(h)),
    "weight left out": ("weighted_expert", lambda f: lambda ff, h, w: ff(h)),
    "gate and up swapped": ("gated_ff", lambda f: lambda x, g, u, d: f(x, u, g, d)),
    "uncapped logits": ("softcap", lambda f: lambda x, cap: x),
}


@pytest.fixture(scope="module")
def mixed_run(tmp_path_factory):
    cfg, w, path = cases.setup(tmp_path_factory.mktemp("mixed"), "mixed", seed=11)
    p = random_prompts([60], cfg["vocab"], seed=2)[0]
    eng = make_engine(path, CPU, F32, max_tokens=64)
    got = eng.feed([(eng.open_sequence(), p, list(range(60)))])
    assert logits_err(got, Oracle(cfg, w).logits(p)) < 2e-4
    return cfg, w, p, got


@pytest.mark.parametrize("fault", [*FAULTS, *FAULTY_FUNCTIONS])
def test_comparison_sees_faults(mixed_run, monkeypatch, fault):
    cfg, w, p, got = mixed_run
    cfg, w = json.loads(json.dumps(cfg)), dict(w)
    if fault in FAULTS:
        FAULTS[fault](cfg, w)
    else:
        name, wrap = FAULTY_FUNCTIONS[fault]
        monkeypatch.setattr(orc, name, wrap(getattr(orc, name)))
    assert logits_err(got, Oracle(cfg, w).logits(p)) > 5e-3, fault


def test_loader_builds_the_configured_model(tmp_path):
    cfg, w, path = cases.setup(tmp_path, "shared_latents", seed=2)
    m = load_pretrained(path, device="cpu", dtype=F32)
    c = m.cfg
    assert isinstance(c, NafazenConfig) and len(c.layers) == 6
    assert [la.mixer.heads for la in c.layers] == [3, 5, 2, 3, 5, 2]
    assert [la.mixer.kv_from for la in c.layers] == [-1, 0, -1, 0, -1, 4]
    assert [la.mixer.rot.scaling is not None for la in c.layers] == [False, False, True, False, False, False]
    assert c.layers[0].moe == MoESpec(5, 2, 40, 56) and c.layers[1].ff == 104 and c.layers[2].ff == 0 and not c.layers[2].moe
    assert c.rms_eps == cfg["norm"]["eps"] and c.embed_scale == 3.7 and c.logit_softcap == 11.0
    assert c.num_params() == sum(v.numel() for v in w.values())
    # one row [latent | rotated key] per token and layer with latents of its own
    assert [(la.n_kv, la.k_dim, la.v_dim) for la in m.cache_layout] == [(1, 128, 0)] * 3
    assert [L["cache"] for L in m.layers] == [0, 0, 1, 0, 2, 2]
    assert c.kv_bytes_per_token() == 3 * 76 * 2 and not m.state_shapes and c.state_bytes_per_seq() == 0
    assert c.eos_ids == (-1,) and c.active_params() < c.num_params()


@pytest.mark.parametrize("change", [lambda d: d["layers"][0].update(type="attention"), lambda d: d.update(extra=1),
                                    lambda d: d["layers"][0]["mixer"].update(mask={"size": 4}),
                                    lambda d: d["layers"][0]["mixer"].update(rot_dim=10),
                                    lambda d: d["layers"][0]["mixer"]["rot"].update(style="halves"),
                                    lambda d: d["layers"][0]["mixer"]["rot"]["scaling"].update(kind="linear"),
                                    lambda d: d["layers"][3]["mixer"].update(kv_from=3),
                                    lambda d: d["layers"][3]["mixer"].update(kv_from=0),
                                    lambda d: d["layers"][2]["mixer"].update(kv_rank=43),
                                    lambda d: d["layers"][1]["mlp"]["router"].update(groups=2),
                                    lambda d: d["layers"][1]["mlp"]["router"].update(top=6),
                                    lambda d: d["layers"][1]["mlp"].update(kind="switch"),
                                    lambda d: d["layers"][0]["mlp"].update(bias=True),
                                    lambda d: d["norm"].update(kind="layer"),
                                    lambda d: d.update(architecture="Other")])
def test_loader_refuses_what_it_does_not_know(tmp_path, change):
    cfg = cases.small_config()
    save_checkpoint(tmp_path, cfg, cases.random_weights(cfg))
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


def test_shared_prefixes_reuse_pages(tmp_path):
    """A prompt that begins like a finished one reads its pages (latents and rotated keys), also in the layers
    that share them, and generates what it does alone."""
    cfg, w, path = cases.setup(tmp_path, "shared_latents", seed=3)
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

    cfg = get_config("nafazen-8b")
    assert 7e9 < cfg.num_params() < 10e9 and cfg.active_params() < 6e9 and plan("nafazen-8b").tensorParallel == 1
    assert len(get_config("nafazen-8b", num_layers=6).layers) == 6
    assert plan("tiny-nafazen").fits
    eng = build_engine("tiny-nafazen", device="cpu", dtype=F32, max_num_seqs=2, max_model_len=64,
                       max_num_batched_tokens=64, num_kv_blocks=16)
    params = SamplingParams(max_tokens=6, temperature=0.8, top_k=20, seed=5, ignore_eos=True)
    out, again = eng.generate([[3, 4, 5]], params), eng.generate([[3, 4, 5]], params)
    assert len(out[0]) == 6 and out == again


def test_trace_runner_program(tmp_path):
    """bin/trace_run end to end: steps on standard input, logits files, requests that end and return."""
    cfg, w, path = cases.setup(tmp_path, "shared_latents", seed=4)
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
            build_model("tiny-nafazen", device="cpu", dtype=F32, pstate=ps)
    finally:
        ps.tp.size = 1
