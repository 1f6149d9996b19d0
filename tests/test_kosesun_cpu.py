"""Kosesun on the CPU: configuration, loader, engine bookkeeping (pages, state slots, portions,
batches) on the reference ops against the plain oracle, and the trace runner."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import kosesun_cases as cases
from hybrid_util import logits_err, make_engine, random_prompts, random_weights, save_checkpoint, small_config
from kosesun_oracle import Oracle
from mlopamd.models import build_model
from mlopamd.models.config import AttentionSpec, GLASpec, HybridConfig, get_config
from mlopamd.models.loader import load_pretrained
from mlopamd.runtime.sampler import SamplingParams

CPU, F32 = torch.device("cpu"), torch.float32
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.mark.parametrize("name", list(cases.CONFIGS))
def test_whole_and_portions(tmp_path, name):
    cases.whole_and_portions(tmp_path, CPU, F32, name, 2e-4)


def test_batches(tmp_path):
    cases.batches(tmp_path, CPU, F32, 2e-4)


def test_long_decoding(tmp_path):
    cases.long_decoding(tmp_path, CPU, F32, 2e-4, n=120)


@pytest.mark.parametrize("tight", [False, True])
def test_greedy_generation(tmp_path, tight):
    cases.greedy_generation(tmp_path, CPU, F32, 1e-3, tight=tight)


def _without(w, *suffixes):
    return {k: v for k, v in w.items() if not k.endswith(suffixes)}


# each mechanism left out or off by a little, in the oracle: the comparison must see it
FAULTS = {
    "sink left out": lambda c, w: w.update({k: torch.full_like(v, -60.0) for k, v in w.items() if k.endswith(".sink")}),
    "sink counted with the scale": lambda c, w: w.update({k: v * c["layers"][0]["mixer"]["scale"] for k, v in w.items() if k.endswith(".sink")}),
    "values not mixed": lambda c, w: w.update({k: torch.zeros_like(v) for k, v in w.items() if k.endswith(".vmix")}),
    "gate left out": lambda c, w: w.update({k: v * 0 + 0 for k, v in w.items() if k.endswith("mix.g")}),
    "rotation one pair short": lambda c, w: [la["mixer"]["rot"].update(dims=la["mixer"]["rot"]["dims"] - 2) for la in c["layers"] if la["type"] == "attention"],
    "rotation base": lambda c, w: [la["mixer"]["rot"].update(base=10000.0) for la in c["layers"] if la["type"] == "attention"],
    "decay constant": lambda c, w: [la["mixer"].update(tau=la["mixer"]["tau"] * 1.2) for la in c["layers"] if la["type"] == "gla"],
    "decay bias left out": lambda c, w: w.update({k: torch.zeros_like(v) for k, v in w.items() if k.endswith(".a2.b")}),
    "stream mix transposed": lambda c, w: w.update({k: v.t().contiguous() for k, v in w.items() if ".hc" in k and k.endswith(".mix")}),
    "soft cap": lambda c, w: c.update(logit_softcap=c["logit_softcap"] * 1.2),
    "norm weights not around zero": lambda c, w: w.update({k: v - 1 for k, v in w.items() if k.endswith((".norm1", ".norm2"))}),
}


@pytest.mark.parametrize("fault", list(FAULTS))
def test_comparison_sees_faults(tmp_path, fault):
    cfg, w, path = cases.setup(tmp_path, "mixed", seed=11)
    p = random_prompts([60], cfg["vocab"], seed=2)[0]
    eng = make_engine(path, CPU, F32, max_tokens=64)
    got = eng.feed([(eng.open_sequence(), p, list(range(60)))])
    assert logits_err(got, Oracle(cfg, w).logits(p)) < 2e-4
    cfg, w = json.loads(json.dumps(cfg)), dict(w)
    FAULTS[fault](cfg, w)
    assert logits_err(got, Oracle(cfg, w).logits(p)) > 5e-3, fault


def test_loader_builds_the_configured_model(tmp_path):
    cfg, w, path = cases.setup(tmp_path, "gla_first", seed=2)
    m = load_pretrained(path, device="cpu", dtype=F32)
    c = m.cfg
    assert isinstance(c, HybridConfig) and c.streams == 2 and len(c.layers) == 5
    assert [type(la.mixer) for la in c.layers] == [GLASpec, GLASpec, AttentionSpec, AttentionSpec, GLASpec]
    assert [bool(la.ff) for la in c.layers] == [True, False, True, False, True]
    assert c.layers[0].mixer.rank == w["l0.mix.a1"].shape[0] and c.rms_eps == cfg["norm"]["eps"]
    assert c.num_params() == sum(v.numel() for k, v in w.items()
                                 if k not in ("l1.norm2", "l3.norm2") and not k.startswith(("l1.hc2", "l3.hc2")))
    assert m.state_shapes == [(2, 20, 12)] * 3 and len(m.cache_layout) == 2
    assert c.eos_ids == (-1,)


@pytest.mark.parametrize("change", [lambda d: d["layers"][0].update(type="window"), lambda d: d.update(extra=1),
                                    lambda d: d["layers"][0]["mixer"].update(window=64),
                                    lambda d: d["layers"][1]["mlp"].update(kind="moe"),
                                    lambda d: d["layers"][0]["mixer"].update(kv_heads=4),
                                    lambda d: d.update(architecture="Other")])
def test_loader_refuses_what_it_does_not_know(tmp_path, change):
    cfg = small_config()
    save_checkpoint(tmp_path, cfg, random_weights(cfg))
    change(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    with pytest.raises((ValueError, KeyError)):
        load_pretrained(tmp_path, device="cpu", dtype=F32)


def test_wrong_tensor_shape_is_refused(tmp_path):
    cfg = small_config()
    w = random_weights(cfg)
    w["l0.mix.sink"] = w["l0.mix.sink"][:-1]
    save_checkpoint(tmp_path, cfg, w)
    with pytest.raises(ValueError, match="l0.mix.sink"):
        load_pretrained(tmp_path, device="cpu", dtype=F32)


def test_presets_build_and_serve():
    from mlopamd.controller.placement import plan
    from mlopamd.runtime.deploy import build_engine

    cfg = get_config("kosesun-8b")
    assert 7.5e9 < cfg.num_params() < 9e9 and plan("kosesun-8b").tensorParallel == 1
    assert len(get_config("kosesun-8b", num_layers=4).layers) == 4
    eng = build_engine("tiny-kosesun", device="cpu", dtype=F32, max_num_seqs=2, max_model_len=64,
                       max_num_batched_tokens=64, num_kv_blocks=16)
    assert get_config("tiny-kosesun").num_params() == sum(
        t.numel() for t in eng.model.weight_tensors()) - sum(  # fused projections and head are padded
        L["proj"].shape[0] * 256 for L in eng.model.layers) - eng.model.head.shape[0] * 256 + _proj_params()
    out = eng.generate([[3, 4, 5]], SamplingParams(max_tokens=6, temperature=0.8, top_k=20, seed=5, ignore_eos=True))
    again = eng.generate([[3, 4, 5]], SamplingParams(max_tokens=6, temperature=0.8, top_k=20, seed=5, ignore_eos=True))
    assert len(out[0]) == 6 and out == again
    assert eng.kv.state_cache.nbytes == 2 * get_config("tiny-kosesun").state_bytes_per_seq()


def _proj_params():
    cfg = get_config("tiny-kosesun")
    n = cfg.vocab_size
    for la in cfg.layers:
        m = la.mixer
        if isinstance(m, AttentionSpec):
            n += (m.heads + m.kv_heads) * m.dim + m.kv_heads * m.vdim + m.heads + 0
        else:
            n += 2 * m.heads * m.dim + 2 * m.heads * m.vdim + m.rank
    # the first mixing layer's share is stored with the checkpoint but not used
    return n * 256 + 1


def test_feed_checks_its_requests(tmp_path):
    cfg, w, path = cases.setup(tmp_path, "mixed")
    eng = make_engine(path, CPU, F32, max_tokens=64)
    s = eng.open_sequence()
    for bad in ([(s, [cfg["vocab"]], [])], [(s, [1, 2], [2])], [(s, [1] * 65, [])]):
        with pytest.raises(ValueError):
            eng.feed(bad)
    assert eng.feed([(s, [1, 2, 3], [])]) is None and s.num_cached == 3
    with pytest.raises(MemoryError):  # the pool holds 64 tokens
        eng.feed([(s, [1] * 40, []), (eng.open_sequence(), [1] * 22, [])])


def test_trace_runner_program(tmp_path):
    """bin/trace_run end to end: steps on standard input, logits files, requests that end and return."""
    cfg, w, path = cases.setup(tmp_path, "gla_first", seed=4)
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
            build_model("tiny-kosesun", device="cpu", dtype=F32, pstate=ps)
    finally:
        ps.tp.size = 1
