"""Lelisun on the CPU engine against the plain oracle."""

import json
import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).resolve().parent))

import lelisun_oracle as oracle  # noqa: E402
from lelisun_common import (  # noqa: E402
    CONFIGS, Case, check_schedules, config, error, run_portions, ssm, write_checkpoint,
)
from llmapigateway_amd.engine import EngineRequest, LLMEngine, SamplingParams  # noqa: E402
from llmapigateway_amd.engine.trace import TraceSession, main as trace_main  # noqa: E402
from llmapigateway_amd.models import HybridModel, get_model_config  # noqa: E402
from llmapigateway_amd.models.weights import open_checkpoint  # noqa: E402


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    root = tmp_path_factory.mktemp("lelisun")
    return {name: Case(name, root / name, seed=i) for i, name in enumerate(CONFIGS)}


@pytest.mark.parametrize("name", list(CONFIGS))
def test_schedules_match_oracle(cases, name):
    check_schedules(cases[name], "cpu", torch.float32, 2e-4)


# ---- the oracle notices what the framework must not get wrong ----
PLANTED = {
    "sink left out": lambda w, c: w.update(
        {k: torch.full_like(t, -30.0) for k, t in w.items() if k.endswith("sink")}),
    "loop step vector": lambda w, c: w.update(
        {"loop.step": w["loop.step"].flip(0)}) if "loop.step" in w else None,
    "last conv tap": lambda w, c: w.update(
        {k: t.roll(1, 1) for k, t in w.items() if k.endswith("mix.conv")}),
}


@pytest.mark.parametrize("what", list(PLANTED))
def test_planted_mistakes_show(cases, what):
    case = cases["odd"]
    toks = case.tokens(60, 5)
    bad = dict(case.weights)
    PLANTED[what](bad, case.cfg)
    assert error(oracle.lelisun(bad, case.cfg, toks), case.expected(toks)) > 0.02


def test_running_maximum_start_shows():
    """m starts at 0: with input gates far below, the denominator's floor is
    e^-m of the real m, not of a maximum that follows the gates from -inf."""
    q = torch.full((3, 1, 2), 0.1, dtype=torch.float64)
    v = torch.ones(3, 1, 2, dtype=torch.float64)
    i = torch.full((3, 1), -4.0, dtype=torch.float64)
    f = torch.full((3, 1), -0.01, dtype=torch.float64)
    y = oracle.mlstm_recurrence(q, q, v, i, f)
    assert y.abs().max() < 0.01  # floor 1 dominates n.q ~ e^-4
    from llmapigateway_amd.ops import reference_hybrid as ref

    segs = type("S", (), dict(cu=torch.tensor([0, 3]), slots=torch.tensor([0])))
    raw = 1e4  # a cap so large that the soft cap is the identity
    fr = f - torch.log(-torch.expm1(f))  # logit of e^f
    gates = torch.cat([i, fr], 1).float()
    got = ref.mlstm(
        (q * 2 ** 0.5).float().view(3, 2), q.float().view(3, 2), v.float().view(3, 2), gates,
        torch.zeros(2), raw, 1, 2, 2, torch.zeros(1, 1, 2, 2), torch.zeros(1, 1, 1, 2),
        torch.zeros(1, 1, 1), torch.arange(3), segs,
    )
    assert torch.allclose(got.double().view(3, 1, 2), y, rtol=1e-3, atol=1e-6)


# ---- generation through the scheduler ----
def greedy(case, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        lg = oracle.lelisun(case.weights, case.cfg, ids)[-1]
        top = lg.topk(2)
        assert top.values[0] - top.values[1] > 1e-4
        ids.append(int(top.indices[0]))
    return ids[len(prompt):]


@pytest.mark.parametrize("name", ["odd", "attention"])
def test_greedy_generation(cases, name):
    case = cases[name]
    prompts = [case.tokens(n, 20 + n) for n in (1, 9, 21)]
    want = [greedy(case, p, 8) for p in prompts]
    # a small prefill budget cuts the prompts and mixes them with decoding
    eng = case.engine("cpu", torch.float32, prefill_budget=5, slots=2)
    reqs = [EngineRequest(p, SamplingParams(max_tokens=8, ignore_eos=True)) for p in prompts]
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
    # a preempted request carries its output over into its prompt
    for r, t, want in zip(reqs, prompts, alone):
        assert r.state == "finished"
        assert (r.prompt_ids + r.out_ids)[len(t):][:24] == want
    assert any(len(r.prompt_ids) > len(t) for r, t in zip(reqs, prompts)), "nothing preempted"


def test_prefix_caching_only_where_pages_are_the_state(cases):
    assert cases["attention"].engine("cpu", torch.float32, prefix_caching=True).prefix_caching
    assert not cases["odd"].engine("cpu", torch.float32, prefix_caching=True).prefix_caching
    case = cases["attention"]
    eng = case.engine("cpu", torch.float32, prefix_caching=True)
    p = SamplingParams(max_tokens=6, ignore_eos=True)
    t = case.tokens(40, 9)
    first = eng.generate(t, p).out_ids
    again = eng.generate(t, SamplingParams(max_tokens=6, ignore_eos=True))
    assert again.num_cached == 32 and again.out_ids == first


def test_sampling_parameters_apply(cases):
    eng = cases["recurrent"].engine("cpu", torch.float32)
    r = eng.generate([1, 2, 3], SamplingParams(max_tokens=3, ignore_eos=True, logit_bias={7: 1e9}))
    assert r.out_ids == [7, 7, 7]
    s = [
        eng.generate([4, 5], SamplingParams(
            max_tokens=6, ignore_eos=True, temperature=1.0, top_k=5, seed=3, logprobs=True,
            top_logprobs=2))
        for _ in range(2)
    ]
    assert s[0].out_ids == s[1].out_ids and len(s[0].out_logprobs) == 6


# ---- configuration, checkpoint, registry ----
def test_checkpoint_reader_and_shapes(cases):
    case = cases["even"]
    f = open_checkpoint(case.path)
    assert set(f.names()) == set(case.weights)
    for name, t in case.weights.items():
        assert torch.equal(f.tensor(name), t)
    cfg = get_model_config(case.path)
    assert HybridModel.tensor_shapes(cfg) == {
        k: tuple(s) for k, s in oracle.tensor_shapes(case.cfg).items()
    }
    assert [r[0] for r in cfg.runs()] == [0] + [1, 2, 3] * 3
    assert [r[1] for r in cfg.runs()] == [None, 0, None, None, 1, None, None, 2, None, None]


def test_checkpoint_errors(tmp_path, cases):
    case = cases["recurrent"]
    w = dict(case.weights)
    del w["l0.mix.f.b"]
    with pytest.raises(KeyError, match="l0.mix.f.b"):
        LLMEngine(model=write_checkpoint(tmp_path / "a", case.cfg, w), dtype=torch.float32,
                  num_blocks=16)
    w["l0.mix.f.b"] = torch.zeros(5, dtype=torch.bfloat16)
    with pytest.raises(ValueError, match="l0.mix.f.b"):
        LLMEngine(model=write_checkpoint(tmp_path / "b", case.cfg, w), dtype=torch.float32,
                  num_blocks=16)
    (tmp_path / "c").mkdir()
    (tmp_path / "c" / "config.json").write_text(json.dumps({"architecture": "Nosuch"}))
    with pytest.raises(KeyError, match="Nosuch"):
        get_model_config(str(tmp_path / "c"))


@pytest.mark.parametrize("change", [
    {"type": "nosuch"}, {"mlp": {"kind": "experts", "ff": 8}},
    {"mixer": dict(heads=6, vdim=4, state=8, groups=4, conv=2, norm_groups=1)},
])
def test_configuration_errors(tmp_path, change):
    cfg = config(32, 64, [dict(ssm(6, 4, 8, 3, 2, 1), **change)])
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(ValueError):
        get_model_config(str(tmp_path))


def test_preset_engine_and_refusals():
    eng = LLMEngine(model="tiny-lelisun", dtype=torch.float32, num_blocks=16, max_batch_size=2)
    r = eng.generate([3, 4, 5], SamplingParams(max_tokens=4, ignore_eos=True))
    assert r.state == "finished" and len(r.out_ids) == 4
    with pytest.raises(ValueError, match="kv_dtype"):
        LLMEngine(model="tiny-lelisun", dtype=torch.float32, num_blocks=16, kv_dtype="fp8")
    with pytest.raises(ValueError, match="float16"):
        LLMEngine(model="tiny-lelisun", dtype=torch.float16, num_blocks=16)
    with pytest.raises(NotImplementedError):
        get_model_config("tiny-lelisun").scaled_for_tp(2)


def test_registry_serves_a_checkpoint_folder(cases):
    import asyncio

    from llmapigateway_amd.config.loader import ProviderDetails
    from llmapigateway_amd.engine.registry import EngineRegistry

    spec = ProviderDetails(baseUrl=f"local://{cases['odd'].path}?device=0").engine_spec()
    assert spec.model == cases["odd"].path
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
    assert sorted(p.name for p in tmp_path.iterdir()) == ["0.f32", "1.f32", "3.f32"]
    V, ea, eb = case.cfg["vocab"], case.expected(a), case.expected(b)
    for step, want in ((0, ea[[0, 19]]), (1, eb[[0]]), (3, torch.stack([ea[29], eb[11]]))):
        got = torch.from_numpy(np.fromfile(tmp_path / f"{step}.f32", dtype="<f4")).view(-1, V)
        assert error(got, want) < 2e-4


def test_trace_session_limits(cases):
    case = cases["attention"]
    ses = TraceSession(case.engine("cpu", torch.float32, blocks=4, slots=2))
    one = [{"id": i, "tokens": [1], "want": []} for i in "ab"]
    ses.step(one)
    with pytest.raises(RuntimeError, match="slot"):
        ses.step([{"id": "c", "tokens": [1], "want": []}])
    with pytest.raises(ValueError):
        ses.step([{"id": "a", "tokens": [case.cfg["vocab"]], "want": []}])
    with pytest.raises(ValueError):
        ses.step([{"id": "a", "tokens": [], "want": []}])
    ses.close("a"), ses.close("b")
    got = run_portions(ses, case, {"c": (case.tokens(50, 1), [50])})
    assert error(got["c"], case.expected(case.tokens(50, 1))) < 2e-4
