"""Duratar on the GPU engine against the plain oracle, fp32 and bf16."""

import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).resolve().parent))

from lelisun_common import check_schedules, error, portions, run_portions  # noqa: E402
from duratar_common import CONFIGS, DuratarCase  # noqa: E402
from llmapigateway_amd import ops  # noqa: E402
from llmapigateway_amd.engine import EngineRequest, LLMEngine, SamplingParams  # noqa: E402
from llmapigateway_amd.engine.trace import TraceSession  # noqa: E402

pytestmark = pytest.mark.gpu

DEV = "cuda:0"


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    assert torch.cuda.is_available() and ops.have_native()
    root = tmp_path_factory.mktemp("duratar")
    return {name: DuratarCase(name, root / name, seed=i) for i, name in enumerate(CONFIGS)}


@pytest.mark.parametrize("name", list(CONFIGS))
def test_schedules_match_oracle_fp32(cases, name):
    check_schedules(cases[name], DEV, torch.float32, 3e-4)


@pytest.mark.parametrize("name", list(CONFIGS))
def test_schedules_in_bf16(cases, name):
    """Every schedule matches the oracle within rounding, wherever prompts are
    cut and whatever else is in the batch."""
    case = cases[name]
    a, b = case.tokens(150, 1), case.tokens(83, 2)
    ses = TraceSession(case.engine(DEV, torch.bfloat16, blocks=24))
    want = case.expected(a)

    def rows(got):
        d = got.double() - want
        d = d - d.mean(-1, keepdim=True)
        return d.pow(2).mean(-1).sqrt() / want.std()

    for sizes in ([150], [86] + [1] * 64, portions(150, [1, 33, 2, 64, 1, 1, 15, 16, 17])):
        e = rows(run_portions(ses, case, {"a": (a, sizes)})["a"])
        assert e.median() < 0.03 and e.max() < 0.12, (sizes[:3], e.median(), e.max())
    jobs = {"a": (a, portions(150, [40, 1, 1, 3])), "b": (b, portions(83, [1, 1, 2, 65]))}
    e = rows(run_portions(ses, case, jobs)["a"])
    assert e.median() < 0.03 and e.max() < 0.12, (e.median(), e.max())


def test_long_prompts_in_bf16(cases):
    """Many chunks of the recurrences, many tiles of the windows."""
    case = cases["even"]
    toks = case.tokens(700, 9)
    want = case.expected(toks)
    ses = TraceSession(case.engine(DEV, torch.bfloat16, blocks=48, max_model_len=768))
    for sizes in ([700], [333, 2, 129, 1, 235]):
        got = run_portions(ses, case, {"a": (toks, sizes)})["a"]
        assert error(got, want) < 0.12


def test_long_decoding(cases):
    """Hundreds of decoded tokens through the captured graph: windows that
    pass over them, pages carried all along."""
    case = cases["odd"]
    toks = case.tokens(330, 8)
    ses = TraceSession(case.engine(DEV, torch.float32, blocks=24, max_model_len=384))
    got = run_portions(ses, case, {"a": (toks, [7] + [1] * 323)})
    assert error(got["a"], case.expected(toks)) < 3e-4
    assert ses.engine.stats["graph_steps"] == 323


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_captured_decode_equals_eager(cases, dtype):
    """Every replay of the decode graphs, with batches that grow and shrink
    over the captured sizes and prompt portions in between, gives the eager
    step's logits."""
    case = cases["even"]
    a, b, c = (case.tokens(n, 60 + n) for n in (60, 45, 33))
    out = []
    for graph in (True, False):
        eng = case.engine(DEV, dtype, use_hipgraph=graph)
        ses = TraceSession(eng)
        jobs = {
            "a": (a, [20] + [1] * 40), "b": (b, [1, 14] + [1] * 30), "c": (c, [3, 1, 1, 20] + [1] * 8),
        }
        out.append(run_portions(ses, case, jobs))
        assert (eng.stats["graph_steps"] > 20) == graph
    for i in "abc":
        assert torch.allclose(out[0][i], out[1][i], atol=1e-4, rtol=1e-4), i


def test_greedy_generation_through_the_scheduler(cases):
    """fp32 on the GPU generates what the CPU engine generates: chunked
    prompts, mixed steps, graph decode with deferred sampling, slot reuse."""
    case = cases["odd"]
    prompts = [case.tokens(n, 20 + n) for n in (1, 9, 40, 21, 70)]

    def run(device):
        eng = case.engine(device, torch.float32, blocks=24, slots=2, prefill_budget=16)
        reqs = [EngineRequest(p, SamplingParams(max_tokens=12, ignore_eos=True)) for p in prompts]
        for r in reqs:
            eng.add_request(r)
        while any(r.state in ("waiting", "running") for r in reqs):
            eng.step()
        assert eng.kv.manager.num_free_blocks == 24
        return [r.out_ids for r in reqs]

    assert run(DEV) == run("cpu")


def test_preset_in_bfloat16():
    eng = LLMEngine(model="tiny-duratar", device=DEV, num_blocks=32, max_batch_size=4)
    reqs = [
        EngineRequest(list(range(3, 3 + n)), SamplingParams(
            max_tokens=10, ignore_eos=True, temperature=t, seed=1))
        for n, t in ((5, 0.0), (64, 0.8), (130, 0.0))
    ]
    for r in reqs:
        eng.add_request(r)
    while any(r.state in ("waiting", "running") for r in reqs):
        eng.step()
    assert all(r.state == "finished" and len(r.out_ids) == 10 for r in reqs)
