"""The flat varlen batch every model's step takes."""

from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import numpy as np
import torch


@dataclass
class ForwardBatch:
    kind: str  # "prefill" | "decode" | "mixed"
    token_ids: torch.Tensor          # [T] int64
    positions: torch.Tensor          # [T] int64
    slot_mapping: torch.Tensor       # [T] int64 (global KV slots; -1 = don't write)
    # prefill:
    cu_seqlens: Optional[torch.Tensor] = None   # [B+1] int32
    max_seqlen: int = 0
    tile_seq: Optional[torch.Tensor] = None     # [ntiles] int32 (GPU kernel tile map)
    tile_off: Optional[torch.Tensor] = None
    # decode:
    block_tables: Optional[torch.Tensor] = None  # [B, max_blocks] int32
    context_lens: Optional[torch.Tensor] = None  # [B] int32
    # prefill with cached prefix (prefix caching): per-seq number of
    # positions already in the paged cache (block_tables set too)
    cached_lens: Optional[torch.Tensor] = None   # [B] int32
    # rows of the flat batch at which logits are needed (last token per seq)
    logits_indices: Optional[torch.Tensor] = None  # [B] int64
    # mixed steps: rows [0, n_prefill_tokens) are prefill (cu_seqlens etc.
    # apply to them), rows [n_prefill_tokens, T) are decode rows with their
    # own tables/lens (decode never shares block_tables with the cached-
    # prefill phase in a mixed step)
    n_prefill_tokens: int = 0
    dec_block_tables: Optional[torch.Tensor] = None  # [Bd, max_blocks] int32
    dec_context_lens: Optional[torch.Tensor] = None  # [Bd] int32
    # models that keep per-sequence state: the same rows seen as segments,
    # one per sequence of the step (a prefill chunk, or one decode row)
    segs: Optional["Segments"] = None


@dataclass
class Segments:
    """The step's rows cut by sequence: segment s is rows cu[s]:cu[s+1] of
    the flat batch, consecutive positions of one sequence, whose recurrent
    state lives in state slot slots[s] (-1: a padding row, nothing of it is
    kept) and whose cache pages are tables[s]. A segment that starts at
    position 0 starts from empty state."""

    cu: torch.Tensor                 # [S+1] int32
    slots: torch.Tensor              # [S] int32
    tables: torch.Tensor             # [S, max_blocks] int32
    row_seg: torch.Tensor            # [T] int32
    block_size: int                  # tokens per cache page
    # host-side twins (absent in captured decode steps, where every
    # segment is one row)
    starts: Optional[np.ndarray] = None   # [S] first position
    lens: Optional[np.ndarray] = None     # [S]
    n_prefill: int = 0                    # the first segments, not decode rows
