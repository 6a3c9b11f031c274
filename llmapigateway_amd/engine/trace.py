"""Externally scheduled runs: a caller says which tokens go through the
engine in which step and reads logits; nothing is sampled.

The sequences use what generation uses: the engine's rows (block table and
recurrent-state slot), its block manager and its two forwards
(LLMEngine._varlen_logits and _decode_logits). A token that continues a
sequence alone is a decode row, anything else a prompt portion; a step of
decode rows only goes through the captured decode graph.

``main`` is bin/trace_run: it reads steps from standard input, one JSON
object a line, and writes the wanted logits of each step to a file.
"""

from __future__ import annotations

import argparse
import dataclasses
import json
import os
import sys
from typing import Dict, List, Optional, Sequence

import numpy as np
import torch

from ..models import MODEL_CLASSES, get_model_config
from ..utils.native_build import ensure_built
from .tokenizer import ByteTokenizer
from .engine import EngineRequest, LLMEngine, SamplingParams


class TraceSession:
    def __init__(self, engine: LLMEngine):
        self.engine = engine
        self._live: Dict[str, EngineRequest] = {}
        self._ntok: Dict[str, int] = {}

    def step(self, entries: Sequence[dict], end: Sequence[str] = ()) -> Optional[torch.Tensor]:
        """entries: [{"id", "tokens", "want"}], all run as one batch; then
        the sequences of ``end`` give back what they hold. Returns the
        logits [wanted, vocab] in the order of entries and of their want
        lists, None if nothing was wanted."""
        eng = self.engine
        vocab = eng.full_config.vocab_size
        spans, dec, at = [], [], []  # at: (is decode row, index) per entry
        seen = set()
        for e in entries:
            if not e["tokens"] or e["id"] in seen:
                raise ValueError(f"entry {e['id']!r}: one non-empty entry per step")
            seen.add(e["id"])
            if min(e["tokens"]) < 0 or max(e["tokens"]) >= vocab:
                raise ValueError(f"entry {e['id']!r}: token out of the vocabulary")
            req = self._live.get(e["id"])
            if req is None:
                if not eng._slot_pool:
                    raise RuntimeError(f"no slot for {e['id']!r}: {len(self._live)} sequences live")
                req = EngineRequest([], SamplingParams())
                eng._claim_slot(req)
                self._live[e["id"]] = req
                self._ntok[e["id"]] = 0
            pos = self._ntok[e["id"]]
            n = pos + len(e["tokens"])
            if n > eng.max_model_len:
                raise RuntimeError(f"{e['id']!r}: {n} tokens exceed {eng.max_model_len}")
            eng._extend_blocks(req, pos, n)
            self._ntok[e["id"]] = n
            if pos and len(e["tokens"]) == 1:
                at.append((True, len(dec)))
                dec.append((req.bt_slot, pos, e["tokens"][0]))
            else:
                at.append((False, len(spans)))
                spans.append((req.bt_slot, pos, e["tokens"]))

        first = np.cumsum([0] + [len(t) for _, _, t in spans])
        want: List[int] = []
        for e, (is_dec, i) in zip(entries, at):
            row0 = int(first[-1]) + i if is_dec else int(first[i])
            want += [row0 + w for w in e.get("want", ())]
        logits = None
        if spans:
            out = eng._varlen_logits(spans, dec, np.asarray(want, dtype=np.int64))
            logits = out if want else None
        elif dec:
            rows, pos, toks = (np.asarray(c, dtype=np.int64) for c in zip(*dec))
            out = eng._decode_logits(rows, pos, toks)
            logits = out[torch.tensor(want, device=out.device)] if want else None

        for rid in end:
            self.close(rid)
        return logits

    def close(self, rid: str) -> None:
        req = self._live.pop(rid)
        del self._ntok[rid]
        if req.block_table:
            self.engine.kv.manager.free(req.block_table)
            req.block_table = []
        self.engine._free_slot(req)


def main(argv: Optional[Sequence[str]] = None) -> int:
    p = argparse.ArgumentParser(
        prog="trace_run",
        description="Replay a trace of token steps through the engine and write logits. "
        "Steps come on standard input, one JSON object a line: "
        '{"step": N, "entries": [{"id", "tokens", "want"}], "end": [ids]}.',
    )
    p.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    p.add_argument("--dtype", required=True, choices=["bfloat16", "float32"])
    p.add_argument("--out", required=True, help="folder for the logits, <step>.f32")
    p.add_argument("--max-tokens", type=int, required=True, help="tokens the cache pool holds")
    p.add_argument("--max-requests", type=int, default=4, help="requests live at a time")
    p.add_argument("--device", default="cuda:0")
    args = p.parse_args(argv)

    config = get_model_config(args.model)
    if args.device.startswith("cuda"):
        ensure_built(MODEL_CLASSES[type(config)].extension)
    torch.set_float32_matmul_precision("highest")
    block = 64
    blocks = max(1, -(-args.max_tokens // block))
    length = blocks * block
    config = dataclasses.replace(config, max_positions=max(config.max_positions, length))
    session = TraceSession(
        LLMEngine(
            model=config, device=args.device, dtype=getattr(torch, args.dtype),
            block_size=block, num_blocks=blocks, max_batch_size=args.max_requests,
            max_model_len=length, tokenizer=ByteTokenizer(config.vocab_size),
        )
    )
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = session.step(step["entries"], step.get("end", ()))
        if logits is not None:
            data = logits.float().cpu().contiguous().numpy().astype("<f4", copy=False)
            data.tofile(os.path.join(args.out, f"{step['step']}.f32"))
        print(f"done {step['step']}", flush=True)
    return 0
