"""Duratar on the CPU engine against the plain oracle."""

import json
import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).resolve().parent))

import duratar_oracle as oracle  # noqa: E402
from lelisun_common import check_schedules, error, run_portions, write_checkpoint  # noqa: E402
from duratar_common import (  # noqa: E402
    CONFIGS, DuratarCase, attn, config, delta, lightning, random_weights, tensor_shapes,
)
from llmapigateway_amd.engine import EngineRequest, LLMEngine, SamplingParams  # noqa: E402
from llmapigateway_amd.engine.kvcache import HybridCache  # noqa: E402
from llmapigateway_amd.engine.trace import TraceSession, main as trace_main  # noqa: E402
from llmapigateway_amd.models import HybridModel, get_model_config  # noqa: E402


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    root = tmp_path_factory.mktemp("duratar")
    return {name: DuratarCase(name, root / name, seed=i) for i, name in enumerate(CONFIGS)}


@pytest.mark.parametrize("name", list(CONFIGS))
def test_schedules_match_oracle(cases, name):
    check_schedules(cases[name], "cpu", torch.float32, 3e-4)


# ---- the oracle notices what the framework must not get wrong ----
def _mixers(c, kind, **kw):
    for layer in c["layers"]:
        if layer["type"] == kind:
            for k, f in kw.items():
                layer["mixer"][k] = f(layer["mixer"])


def _mask(c, **kw):
    _mixers(c, "attention", mask=lambda m: {
        k: max(kw.get(k, lambda x: x)(v), 1 if k == "size" else 0) for k, v in m["mask"].items()})


def _leaf(w, leaf, f):
    w.update({k: f(t.float()).to(t.dtype) for k, t in w.items() if k.endswith(leaf)})


def _rot(c, **kw):
    _mixers(c, "attention", rot=lambda m: dict(m["rot"], **kw))


PLANTED = {
    "window one longer": lambda w, c: _mask(c, size=lambda x: x + 1),
    "window one shorter": lambda w, c: _mask(c, size=lambda x: x - 1),
    "one more token kept": lambda w, c: _mask(c, keep_first=lambda x: x + 1),
    "one token less kept": lambda w, c: _mask(c, keep_first=lambda x: x - 1),
    "nothing kept": lambda w, c: _mask(c, keep_first=lambda x: 0),
    "rotation base": lambda w, c: _rot(c, base=200.0),
    "rotated dimensions": lambda w, c: _rot(c, dims=8),
    "frequency scaling": lambda w, c: _rot(c, scaling=None),
    "scaling factor": lambda w, c: _rot(c, scaling=dict(factor=2.0, low=1.0, high=6.0, original=64)),
    "scaling's upper end": lambda w, c: _rot(
        c, scaling=dict(factor=5.0, low=1.0, high=4.0, original=64)),
    "difference of the maps": lambda w, c: _mixers(c, "attention", diff=lambda m: m["diff"] + 0.1),
    "lambda's vectors": lambda w, c: _leaf(w, "lq1", lambda t: t * 0),
    "lambda's second vectors": lambda w, c: _leaf(w, "lk2", lambda t: t * 0),
    "score scale": lambda w, c: _mixers(c, "attention", scale=lambda m: m["scale"] * 1.1),
    "query norm": lambda w, c: _leaf(w, "q.norm", lambda t: t * 0 + 1),
    "key norm": lambda w, c: _leaf(w, "k.norm", lambda t: t * 0 + 1),
    "lightning decay": lambda w, c: _mixers(
        c, "lightning", decay=lambda m: [x * 0.97 for x in m["decay"]]),
    "lightning gate": lambda w, c: _leaf(w, "l3.mix.g", lambda t: t * 0),
    "lightning norm": lambda w, c: _leaf(w, "l3.mix.norm", lambda t: t * 0 + 1),
    "taps reversed": lambda w, c: _leaf(w, ".conv", lambda t: t.flip(1)),
    "write strength": lambda w, c: _leaf(w, "l1.mix.b", lambda t: t * 0),
    "decay rate": lambda w, c: _leaf(w, "A_log", lambda t: t + 0.3),
    "decay bias": lambda w, c: _leaf(w, "dt_bias", lambda t: t + 0.5),
    "decay projection": lambda w, c: _leaf(w, "a2", lambda t: t * 0),
    "delta gate": lambda w, c: _leaf(w, "g2", lambda t: t * 0),
    "delta norm": lambda w, c: _leaf(w, "l1.mix.norm", lambda t: t * 0 + 1),
    "activation's upper half": lambda w, c: _leaf(w, "act", lambda t: t + torch.tensor([0.3, 0.])),
    "activation's lower half": lambda w, c: _leaf(w, "act", lambda t: t + torch.tensor([0., 0.5])),
    "layer scale": lambda w, c: _leaf(w, "ls1", lambda t: t * 0 + 1),
    "second layer scale": lambda w, c: _leaf(w, "ls2", lambda t: t * 0 + 1),
    "streams' mix transposed": lambda w, c: _leaf(w, "hc1.mix", lambda t: t.T.contiguous()),
    "what is read": lambda w, c: _leaf(w, "hc2.in", lambda t: t * 0 + 1 / 3),
    "what is written": lambda w, c: _leaf(w, "hc1.out", lambda t: t * 0 + 1),
    "norm's number": lambda w, c: _leaf(w, "norm2", lambda t: t * 0 + 1),
    "the embedding's norm": lambda w, c: _leaf(w, "embed.norm", lambda t: t * 2),
    "norm epsilon": lambda w, c: c["norm"].update(eps=0.1),
    "another layer's keys": lambda w, c: (
        c["layers"][2]["mixer"].pop("kv_from"),
        w.update({f"l2.mix.{n}": w[f"l0.mix.{n}"].flip(0) for n in ("k", "v", "k.norm")})),
}


@pytest.mark.parametrize("what", list(PLANTED))
def test_planted_mistakes_show(cases, what):
    case = cases["odd"]
    toks = case.tokens(90, 5)
    bad, cfg = dict(case.weights), json.loads(json.dumps(case.cfg))
    PLANTED[what](bad, cfg)
    assert error(oracle.duratar(bad, cfg, toks), case.expected(toks)) > 0.008


# ---- generation through the scheduler ----
def greedy(case, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        lg = oracle.duratar(case.weights, case.cfg, ids)[-1]
        top = lg.topk(2)
        assert top.values[0] - top.values[1] > 1e-4
        ids.append(int(top.indices[0]))
    return ids[len(prompt):]


@pytest.mark.parametrize("name", ["odd", "recurrent", "attention"])
def test_greedy_generation(cases, name):
    case = cases[name]
    prompts = [case.tokens(n, 20 + n) for n in (1, 9, 45)]
    want = [greedy(case, p, 6) for p in prompts]
    # a small prefill budget cuts the prompts and mixes them with decoding
    eng = case.engine("cpu", torch.float32, prefill_budget=5, slots=2)
    reqs = [EngineRequest(p, SamplingParams(max_tokens=6, ignore_eos=True)) for p in prompts]
    for r in reqs:
        eng.add_request(r)
    while any(r.state in ("waiting", "running") for r in reqs):
        eng.step()
    assert [r.out_ids for r in reqs] == want
    if not eng.prefix_caching:
        assert eng.kv.manager.num_free_blocks == 40


def test_prefix_caching(cases):
    """Pages are an attention-only model's whole state, also where a layer
    reads another one's."""
    case = cases["attention"]
    head = case.tokens(48, 50)
    prompts = [head + case.tokens(n, 51 + n) for n in (5, 9)]
    p = SamplingParams(max_tokens=5, ignore_eos=True)
    want = [case.engine("cpu", torch.float32).generate(t, p).out_ids for t in prompts]
    eng = case.engine("cpu", torch.float32, prefix_caching=True)
    assert eng.prefix_caching
    reqs = [eng.generate(t, p) for t in prompts]
    assert [r.out_ids for r in reqs] == want
    assert [r.num_cached for r in reqs] == [0, 48]
    assert not cases["odd"].engine("cpu", torch.float32, prefix_caching=True).prefix_caching


def test_preempted_request_restarts(cases):
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


# ---- configuration, checkpoint, cache, registry ----
def test_checkpoint_shapes_and_runs(cases):
    for name, case in cases.items():
        cfg = get_model_config(case.path)
        assert HybridModel.tensor_shapes(cfg) == tensor_shapes(case.cfg)
        assert cfg.streams == case.cfg["streams"] and cfg.scalar_norms and cfg.layer_scale
    cfg = get_model_config(cases["odd"].path)
    assert [cfg.kv_source(i) for i in range(5)] == [0, 1, 0, 3, 0]


def test_layers_that_share_keys_share_pages(cases):
    cfg = get_model_config(cases["odd"].path)
    c = HybridCache(cfg, 4, 16, "cpu", torch.float32, num_slots=2)
    assert c.runs[2] is c.runs[0] and c.runs[4] is c.runs[0] and set(c.runs[0]) == {"k", "v"}
    row = 3 * (2 * 18 + 26)
    assert HybridCache.block_bytes(cfg, 16, torch.float32) == 16 * row * 4


def test_checkpoint_errors(tmp_path, cases):
    case = cases["attention"]
    w = dict(case.weights)
    w["l0.hc1.mix"] = w["l0.hc1.mix"][:, :-1].contiguous()
    with pytest.raises(ValueError, match="hc1.mix"):
        LLMEngine(model=write_checkpoint(tmp_path / "a", case.cfg, w), dtype=torch.float32,
                  num_blocks=16)
    del w["l0.hc1.mix"]
    with pytest.raises(KeyError, match="hc1.mix"):
        LLMEngine(model=write_checkpoint(tmp_path / "b", case.cfg, w), dtype=torch.float32,
                  num_blocks=16)


OK = attn(4, 2, 8, 8, 5, 1, 4)


@pytest.mark.parametrize("layers,streams", [
    ([attn(6, 4, 8, 8, 5, 1, 4)], 2),                           # 4 does not divide 6
    ([attn(4, 2, 8, 8, 0, 1, 4)], 2),                           # no window
    ([attn(4, 2, 8, 8, 5, 1, 10)], 2),                          # rotates more than there is
    ([attn(4, 2, 8, 8, 5, 1, 3)], 2),                           # half a pair
    ([delta(3, 2, 8, 8, 4, 4, 4)], 2),                          # 2 does not divide 3
    ([lightning(3, 8, 8, (0.9, 0.8))], 2),                      # a decay is missing
    ([lightning(1, 8, 8, (1.5,))], 2),                          # it would grow
    ([OK], 17), ([OK], 0),                                      # streams
    ([OK, attn(4, 2, 8, 8, 5, 1, 4, kv_from=1)], 2),            # its own
    ([attn(4, 2, 8, 8, 5, 1, 4, kv_from=1), OK], 2),            # a later one's
    ([OK, attn(4, 4, 8, 8, 5, 1, 4, kv_from=0)], 2),            # another number of heads
    ([OK, attn(4, 2, 8, 8, 5, 1, 4, kv_from=0, base=9.0)], 2),  # another rotation
    ([OK, attn(4, 2, 8, 8, 5, 1, 4, kv_from=0), attn(4, 2, 8, 8, 5, 1, 4, kv_from=1)], 2),
    ([lightning(1, 8, 8, (0.5,)), attn(4, 2, 8, 8, 5, 1, 4, kv_from=0)], 2),
    ([dict(OK, mlp={"kind": "nosuch", "ff": 8})], 2),
    ([dict(OK, type="nosuch")], 2),
])
def test_configuration_errors(tmp_path, layers, streams):
    ok = [dict(x, mlp=None, type=x["type"] if x["type"] != "nosuch" else "attention")
          for x in layers]
    path = write_checkpoint(tmp_path / "m", config(32, 64, streams, layers),
                            random_weights(config(32, 64, max(streams, 1), ok)))
    with pytest.raises(ValueError):
        get_model_config(path)


def test_preset_engine_and_refusals():
    eng = LLMEngine(model="tiny-duratar", dtype=torch.float32, num_blocks=16, max_batch_size=2)
    r = eng.generate([3, 4, 5], SamplingParams(max_tokens=4, ignore_eos=True))
    assert r.state == "finished" and len(r.out_ids) == 4
    with pytest.raises(ValueError, match="kv_dtype"):
        LLMEngine(model="tiny-duratar", dtype=torch.float32, num_blocks=16, kv_dtype="fp8")
    with pytest.raises(NotImplementedError):
        get_model_config("tiny-duratar").scaled_for_tp(2)


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
    a, b = case.tokens(60, 41), case.tokens(12, 42)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:41], "want": [0, 40]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[:1], "want": [0]},
                                {"id": "a", "tokens": a[41:42], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": a[42:43], "want": []}], "end": []},
        {"step": 3, "entries": [{"id": "a", "tokens": a[43:], "want": [16]},
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
    for step, want in ((0, ea[[0, 40]]), (1, eb[[0]]), (3, torch.stack([ea[59], eb[11]]))):
        got = torch.from_numpy(np.fromfile(tmp_path / f"{step}.f32", dtype="<f4")).view(-1, V)
        assert error(got, want) < 3e-4


@pytest.mark.parametrize("name", ["odd", "recurrent"])
def test_slots_and_pages_of_a_closed_sequence_are_clean(cases, name):
    """Another sequence in a used slot and used pages gives what it gives in a
    fresh engine."""
    case = cases[name]
    ses = TraceSession(case.engine("cpu", torch.float32, blocks=6, slots=1))
    a, b = case.tokens(90, 1), case.tokens(40, 2)
    run_portions(ses, case, {"a": (a, [60, 1, 29])})
    got = run_portions(ses, case, {"b": (b, [1, 2, 37])})
    assert error(got["b"], case.expected(b)) < 3e-4


def test_the_first_tokens_alone(cases):
    """A sequence of one to five tokens, whole and token by token."""
    for name, case in cases.items():
        for n in range(1, 6):
            toks = case.tokens(n, 70 + n)
            ses = TraceSession(case.engine("cpu", torch.float32))
            for sizes in ([n], [1] * n):
                got = run_portions(ses, case, {"a": (toks, sizes)})
                assert error(got["a"], case.expected(toks)) < 3e-4, (name, n)
