"""Externally scheduled runs: a caller says which tokens go through the
engine in which step and reads logits; nothing is sampled.

The sequences use what generation uses: the engine's rows (block table and
recurrent-state slot), its block manager and its two forwards
(LLMEngine._varlen_logits and _decode_logits). A token that continues a
sequence alone is a decode row, anything else a prompt portion; a step of
decode rows only goes through the captured decode graph.
"""

from __future__ import annotations

from typing import Dict, List, Optional, Sequence

import numpy as np
import torch

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
        spans, dec, at = [], [], []  # at: (is decode row, index) per entry
        seen = set()
        for e in entries:
            if not e["tokens"] or e["id"] in seen:
                raise ValueError(f"entry {e['id']!r}: one non-empty entry per step")
            seen.add(e["id"])
            vocab = eng.full_config.vocab_size
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
