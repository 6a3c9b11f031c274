"""Small Lelisun configurations, a checkpoint writer and step drivers shared
by the CPU and GPU tests."""

from __future__ import annotations

import json
import struct

import torch

from lelisun_oracle import lelisun, random_weights
from llmapigateway_amd.engine import LLMEngine
from llmapigateway_amd.engine.trace import TraceSession


def attn(heads, dim, rot, vdim, kv, q, mult=2.0, base=10000.0, ff=None):
    # a scale above 1/sqrt(d) makes single keys stand out in the softmax
    return {
        "type": "latent_attention",
        "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": kv,
                  "q_rank": q, "scale": mult * (dim + rot) ** -0.5,
                  "rot": {"base": base, "dims": rot}},
        "mlp": {"kind": "dense", "ff": ff} if ff else None,
    }


def ssm(heads, vdim, state, groups, conv, norm_groups, ff=None):
    return {
        "type": "mamba2",
        "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
                  "conv": conv, "norm_groups": norm_groups},
        "mlp": {"kind": "dense", "ff": ff} if ff else None,
    }


def mem(heads, dim, vdim, cap, ff=None):
    return {
        "type": "mlstm",
        "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap},
        "mlp": {"kind": "dense", "ff": ff} if ff else None,
    }


def config(width, vocab, layers, loop=None, eps=1e-5, scale=3.0):
    return {
        "architecture": "Lelisun", "width": width, "vocab": vocab, "layers": layers,
        "embedding": {"scale": scale}, "norm": {"eps": eps},
        "loop": dict(zip(("start", "stop", "times"), loop)) if loop else None,
    }


CONFIGS = {
    # sizes that are no multiples of anything: the any-size kernels
    "odd": config(
        70, 211,
        [ssm(6, 10, 22, 3, 3, 2, ff=54), attn(3, 18, 6, 26, 34, 42), mem(3, 14, 22, 5.0, ff=50)],
        loop=(1, 3, 2), eps=1e-4, scale=5.5,
    ),
    # multiples of 8: the MFMA kernels, several tiles and slices of each
    "even": config(
        128, 300,
        [attn(20, 32, 16, 40, 136, 72, ff=96), mem(2, 136, 200, 15.0),
         ssm(6, 72, 88, 2, 4, 3), attn(5, 40, 24, 72, 64, 48, base=500.0)],
        loop=(1, 4, 3), eps=1e-5, scale=2.0,
    ),
    # recurrent layers only, no loop, a one-tap convolution
    "recurrent": config(
        96, 180, [mem(4, 24, 16, 8.0), ssm(4, 16, 32, 4, 1, 1, ff=64)], eps=1e-3, scale=1.0,
    ),
    # attention only, looped once, from the first layer on
    "attention": config(
        64, 190, [attn(4, 16, 8, 24, 48, 40, ff=72), attn(2, 24, 4, 16, 32, 56)],
        loop=(0, 1, 1), scale=8.0,
    ),
}

_DTYPE = {torch.bfloat16: "BF16", torch.float32: "F32", torch.int32: "I32"}


def write_checkpoint(folder, cfg, weights):
    """config.json + model.safetensors in ``folder``."""
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    header, blobs, at = {}, [], 0
    for name, t in weights.items():
        raw = t.contiguous().reshape(-1).view(torch.uint8).numpy().tobytes()
        header[name] = {"dtype": _DTYPE[t.dtype], "shape": list(t.shape),
                        "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    h = json.dumps(header).encode()
    (folder / "model.safetensors").write_bytes(struct.pack("<Q", len(h)) + h + b"".join(blobs))
    return str(folder)


class Case:
    """A configuration with weights on disk, and the oracle's logits."""

    def __init__(self, name, folder, seed=0):
        self.cfg = CONFIGS[name]
        self.weights = random_weights(self.cfg, seed)
        self.path = write_checkpoint(folder, self.cfg, self.weights)
        self._logits = {}

    def tokens(self, n, seed):
        g = torch.Generator().manual_seed(seed)
        return torch.randint(0, self.cfg["vocab"], (n,), generator=g).tolist()

    def expected(self, tokens):
        key = tuple(tokens)
        if key not in self._logits:
            self._logits[key] = lelisun(self.weights, self.cfg, tokens)
        return self._logits[key]

    def engine(self, device, dtype, blocks=40, slots=4, block_size=16, **kw):
        return LLMEngine(
            model=self.path, device=device, dtype=dtype, num_blocks=blocks,
            max_batch_size=slots, block_size=block_size,
            max_model_len=kw.pop("max_model_len", blocks * block_size), **kw,
        )


def error(got, want):
    """Worst row: rms difference of the centred logits over their rms."""
    d = got.double().cpu() - want
    d = d - d.mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / want.std()).max())


def run_portions(session, case, jobs):
    """jobs: {id: (tokens, [portion sizes])}, one portion of every job per
    step; returns {id: logits of all its tokens}. Finished jobs are closed."""
    at = {i: 0 for i in jobs}
    sizes = {i: list(s) for i, (_, s) in jobs.items()}
    out = {i: [] for i in jobs}
    while any(sizes.values()):
        entries, end = [], []
        for i, (toks, _) in jobs.items():
            if not sizes[i]:
                continue
            n = sizes[i].pop(0)
            entries.append({"id": i, "tokens": toks[at[i] : at[i] + n], "want": list(range(n))})
            at[i] += n
            if not sizes[i]:
                assert at[i] == len(toks)
                end.append(i)
        lg, r = session.step(entries, end), 0
        for e in entries:
            n = len(e["tokens"])
            out[e["id"]].append(lg[r : r + n].cpu())
            r += n
    return {i: torch.cat(v) for i, v in out.items()}


def portions(n, pattern):
    """Cut n tokens by a repeating pattern of sizes."""
    out, k = [], 0
    while sum(out) < n:
        out.append(min(pattern[k % len(pattern)], n - sum(out)))
        k += 1
    return out


def check_schedules(case, device, dtype, limit):
    """Whole prompts, token by token, portions, unequal batches and reuse of
    pages and slots, all against the oracle."""
    a, b, c = case.tokens(150, 1), case.tokens(83, 2), case.tokens(17, 3)
    eng = case.engine(device, dtype, blocks=24)
    ses = TraceSession(eng)
    plans = {
        "whole": [150],
        "decode": [86] + [1] * 64,
        "from the start": [1] * 20 + [130],
        "twos and threes": portions(150, [2, 3]),
        "uneven": portions(150, [1, 33, 2, 64, 1, 1, 15, 16, 17]),
    }
    for name, sizes in plans.items():
        got = run_portions(ses, case, {"a": (a, sizes)})
        assert error(got["a"], case.expected(a)) < limit, name
    jobs = {
        "a": (a, portions(150, [40, 1, 1, 3])), "b": (b, portions(83, [1, 1, 2, 65])),
        "c": (c, portions(17, [5])),
    }
    got = run_portions(ses, case, jobs)
    for i, (toks, _) in jobs.items():
        assert error(got[i], case.expected(toks)) < limit, i
    assert eng.kv.manager.num_free_blocks == 24 and len(eng._slot_pool) == 4
