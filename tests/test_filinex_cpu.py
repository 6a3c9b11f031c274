"""Filinex on the CPU engine against the plain oracle."""

import json
import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).resolve().parent))

import filinex_oracle as oracle  # noqa: E402
from filinex_common import (  # noqa: E402
    CONFIGS, FilinexCase, config, moe, par, random_weights, tensor_shapes, wkv,
)
from lelisun_common import check_schedules, error, run_portions, write_checkpoint  # noqa: E402
from llmapigateway_amd.engine import EngineRequest, LLMEngine, SamplingParams  # noqa: E402
from llmapigateway_amd.engine.trace import TraceSession, main as trace_main  # noqa: E402
from llmapigateway_amd.models import HybridModel, get_model_config  # noqa: E402


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    root = tmp_path_factory.mktemp("filinex")
    return {name: FilinexCase(name, root / name, seed=i) for i, name in enumerate(CONFIGS)}


@pytest.mark.parametrize("name", list(CONFIGS))
def test_schedules_match_oracle(cases, name):
    check_schedules(cases[name], "cpu", torch.float32, 2e-4)


# ---- the oracle notices what the framework must not get wrong ----
def _set(c, *path_value):
    *path, key, value = path_value
    for p in path:
        c = c[p]
    c[key] = value


PLANTED = {
    "sink left out": lambda w, c: w.update(
        {k: torch.full_like(t, -30.0) for k, t in w.items() if k.endswith("sink")}),
    "score cap": lambda w, c: _set(c, "layers", 1, "mixer", "left", "softcap", 1e6),
    "logit cap": lambda w, c: _set(c, "logit_softcap", 1e6),
    "tau": lambda w, c: _set(c, "layers", 1, "mixer", "right", "tau", 1.0),
    "side scales": lambda w, c: _set(c, "layers", 1, "mixer", "left_scale", 1.0),
    "attention gate": lambda w, c: w.update(
        {k: t * 0 for k, t in w.items() if k.endswith("left.g")}),
    "expert limit": lambda w, c: _set(c, "layers", 0, "mlp", "expert", "limit", 100.0),
    "shared limit": lambda w, c: _set(c, "layers", 0, "mlp", "shared", "limit", 100.0),
    "router bias": lambda w, c: w.update(
        {k: -2 * t for k, t in w.items() if k.endswith("router.b")}),
    "bonus": lambda w, c: w.update({k: t * 0 for k, t in w.items() if k.endswith("mix.u")}),
    "token shift": lambda w, c: w.update({k: t * 0 for k, t in w.items() if ".mu." in k}),
    "norm of a sublayer's output": lambda w, c: w.update(
        {k: t * 2 for k, t in w.items() if k.endswith("norm1b.alpha")}),
    "loop input": lambda w, c: w.update({"loop.in": w["loop.in"].flip(1)}),
    "passes": lambda w, c: _set(c, "loop", "times", 3),
}


@pytest.mark.parametrize("what", list(PLANTED))
def test_planted_mistakes_show(cases, what):
    case = cases["odd"]
    toks = case.tokens(60, 5)
    bad, cfg = dict(case.weights), json.loads(json.dumps(case.cfg))
    PLANTED[what](bad, cfg)
    assert error(oracle.filinex(bad, cfg, toks), case.expected(toks)) > 0.02


# ---- generation through the scheduler ----
def greedy(case, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        lg = oracle.filinex(case.weights, case.cfg, ids)[-1]
        top = lg.topk(2)
        assert top.values[0] - top.values[1] > 1e-4
        ids.append(int(top.indices[0]))
    return ids[len(prompt):]


@pytest.mark.parametrize("name", ["odd", "plain"])
def test_greedy_generation(cases, name):
    case = cases[name]
    prompts = [case.tokens(n, 20 + n) for n in (1, 9, 21)]
    want = [greedy(case, p, 6) for p in prompts]
    # a small prefill budget cuts the prompts and mixes them with decoding
    eng = case.engine("cpu", torch.float32, prefill_budget=5, slots=2)
    reqs = [EngineRequest(p, SamplingParams(max_tokens=6, ignore_eos=True)) for p in prompts]
    for r in reqs:
        eng.add_request(r)
    while any(r.state in ("waiting", "running") for r in reqs):
        eng.step()
    assert [r.out_ids for r in reqs] == want
    assert eng.kv.manager.num_free_blocks == 40


def test_preempted_request_restarts_from_empty_state(cases):
    case = cases["odd"]
    prompts = [case.tokens(20, 31), case.tokens(18, 32)]
    p = SamplingParams(max_tokens=24, ignore_eos=True)
    alone = [case.engine("cpu", torch.float32).generate(t, p).out_ids for t in prompts]
    eng = case.engine("cpu", torch.float32, blocks=5, max_model_len=64)
    reqs = [EngineRequest(t, SamplingParams(max_tokens=24, ignore_eos=True)) for t in prompts]
    for r in reqs:
        eng.add_request(r)
    for _ in range(400):
        if all(r.state == "finished" for r in reqs):
            break
        eng.step()
    for r, t, want in zip(reqs, prompts, alone):
        assert r.state == "finished"
        assert (r.prompt_ids + r.out_ids)[len(t):][:24] == want
    assert any(len(r.prompt_ids) > len(t) for r, t in zip(reqs, prompts)), "nothing preempted"


def test_prefix_caching_is_off(cases):
    """Pages are not a sequence's whole state where layers are recurrent."""
    assert not cases["plain"].engine("cpu", torch.float32, prefix_caching=True).prefix_caching


# ---- configuration, checkpoint, registry ----
def test_checkpoint_shapes_and_runs(cases):
    case = cases["even"]
    cfg = get_model_config(case.path)
    assert HybridModel.tensor_shapes(cfg) == tensor_shapes(case.cfg)
    assert [r[0] for r in cfg.runs()] == [0, 1] * 3 + [2]
    assert [r[1] for r in cfg.runs()] == [0, None, 1, None, 2, None, None]
    assert cfg.norm == "tanh" and cfg.logit_softcap == 30.0


def test_checkpoint_errors(tmp_path, cases):
    case = cases["recurrent"]
    w = dict(case.weights)
    w["l0.mlp.router"] = w["l0.mlp.router"][:, :-1].contiguous()
    with pytest.raises(ValueError, match="router"):
        LLMEngine(model=write_checkpoint(tmp_path / "a", case.cfg, w), dtype=torch.float32,
                  num_blocks=16)
    del w["l0.mlp.router"]
    with pytest.raises(KeyError, match="router"):
        LLMEngine(model=write_checkpoint(tmp_path / "b", case.cfg, w), dtype=torch.float32,
                  num_blocks=16)


@pytest.mark.parametrize("layer", [
    par(6, 4, 8, 8, 5.0, 2, 8, 8, 4.0, (1, 1), 4),                        # 4 does not divide 6
    par(4, 2, 8, 8, 0.0, 2, 8, 8, 4.0, (1, 1), 4),                        # no cap
    wkv(2, 16, 4, moe(3, 4, 8, 1.0, 8, 1.0)),                             # 4 of 3 experts
    dict(wkv(2, 16, 4), mlp={"kind": "nosuch"}),
])
def test_configuration_errors(tmp_path, layer):
    cfg = config(32, 64, [layer])
    ok = config(32, 64, [dict(layer, mlp=None)])
    path = write_checkpoint(tmp_path / "m", cfg, random_weights(ok))
    with pytest.raises(ValueError):
        get_model_config(path)


def test_preset_engine_and_refusals():
    eng = LLMEngine(model="tiny-filinex", dtype=torch.float32, num_blocks=16, max_batch_size=2)
    r = eng.generate([3, 4, 5], SamplingParams(max_tokens=4, ignore_eos=True))
    assert r.state == "finished" and len(r.out_ids) == 4
    with pytest.raises(ValueError, match="kv_dtype"):
        LLMEngine(model="tiny-filinex", dtype=torch.float32, num_blocks=16, kv_dtype="fp8")
    with pytest.raises(NotImplementedError):
        get_model_config("tiny-filinex").scaled_for_tp(2)


def test_registry_serves_a_checkpoint_folder(cases):
    import asyncio

    from llmapigateway_amd.config.loader import ProviderDetails
    from llmapigateway_amd.engine.registry import EngineRegistry

    spec = ProviderDetails(baseUrl=f"local://{cases['odd'].path}?device=0").engine_spec()
    reg = EngineRegistry()

    async def ask():
        try:
            return await reg.make_request(
                "p", spec, {"prompt": "hi", "max_tokens": 5, "ignore_eos": True}, False)
        finally:
            await reg.aclose()

    body, err = asyncio.run(ask())
    assert err is None and body["usage"]["completion_tokens"] == 5


# ---- external schedules ----
def test_trace_run_program(cases, tmp_path, monkeypatch, capsys):
    import io

    import numpy as np

    case = cases["odd"]
    a, b = case.tokens(30, 41), case.tokens(12, 42)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [0, 19]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[:1], "want": [0]},
                                {"id": "a", "tokens": a[20:21], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": a[21:22], "want": []}], "end": []},
        {"step": 3, "entries": [{"id": "a", "tokens": a[22:], "want": [7]},
                                {"id": "b", "tokens": b[1:], "want": [10]}], "end": ["a", "b"]},
    ]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(map(json.dumps, steps)) + "\n"))
    rc = trace_main(["--model", case.path, "--dtype", "float32", "--out", str(tmp_path),
                     "--max-tokens", "128", "--device", "cpu"])
    assert rc == 0
    assert [x for x in capsys.readouterr().out.splitlines() if x.startswith("done")] == [
        f"done {i}" for i in range(4)
    ]
    V, ea, eb = case.cfg["vocab"], case.expected(a), case.expected(b)
    for step, want in ((0, ea[[0, 19]]), (1, eb[[0]]), (3, torch.stack([ea[29], eb[11]]))):
        got = torch.from_numpy(np.fromfile(tmp_path / f"{step}.f32", dtype="<f4")).view(-1, V)
        assert error(got, want) < 2e-4


def test_slots_and_pages_of_a_closed_sequence_are_clean(cases):
    """Another sequence in a used slot and used pages gives what it gives in
    a fresh engine."""
    case = cases["plain"]
    ses = TraceSession(case.engine("cpu", torch.float32, blocks=6, slots=1))
    a, b = case.tokens(90, 1), case.tokens(40, 2)
    run_portions(ses, case, {"a": (a, [60, 1, 29])})
    got = run_portions(ses, case, {"b": (b, [1, 2, 37])})
    assert error(got["b"], case.expected(b)) < 2e-4
