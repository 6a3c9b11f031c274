"""Hyper-connected residual streams.

Instead of one residual stream there are S copies of it. Sublayer q reads
u = sum_s in_q[s] x_s and, with y its output, all streams become

    x_t <- sum_s mix_q[s, t] x_s + out_q[t] y

All of this is linear in the stored streams and in the outputs y since, so the
streams need not be rewritten after every sublayer: up to ``DEFER`` outputs
stay pending, and what a sublayer reads is one combination of stored streams
and pending outputs whose coefficients are made here, once, in float64. Only
the first sublayers of a step see a single stored stream: all copies start
equal.
"""

from __future__ import annotations

from typing import List, NamedTuple, Optional, Tuple

import torch

from .. import ops

DEFER = 4  # pending outputs from which reading them again costs what a rewrite does


class Read(NamedTuple):
    """coef [stored + pending, columns] fp32: the first column is what the
    sublayer reads; with ``rewrite`` the others are the new streams."""

    coef: torch.Tensor
    rewrite: bool


class HyperStreams:
    def __init__(self, streams: int, subs: List[Tuple[torch.Tensor, ...]], device):
        """subs: (in [S], mix [S, S], out [S]) of every sublayer in order."""
        S = streams
        self.reads: List[Read] = []
        base = torch.ones(1, S, dtype=torch.float64)         # stored -> streams
        pending = torch.zeros(0, S, dtype=torch.float64)     # outputs -> streams
        ends = [(torch.ones(S, dtype=torch.float64), None, None)]  # the last: their sum
        for w_in, mix, w_out in [tuple(t.double().cpu() for t in s) for s in subs] + ends:
            rows = torch.cat([base, pending])
            read = rows @ w_in[:, None]
            rewrite = len(pending) >= DEFER and mix is not None
            self.reads.append(Read(
                (torch.cat([read, rows], 1) if rewrite else read).float().contiguous().to(device),
                rewrite,
            ))
            if mix is None:
                break
            if rewrite:
                base, pending = torch.eye(S, dtype=torch.float64), pending[:0]
            base = base @ mix
            pending = torch.cat([pending @ mix, w_out[None]])

    def read(self, q: int, x: torch.Tensor, pending: list, norm: torch.Tensor, eps: float, dtype,
             rows: Optional[torch.Tensor] = None):
        """The normed input of sublayer q (the last q: of the head), from the
        stored streams x [T, 1 or S, W] and the pending (output, scale [W] or
        None) pairs; returns it, the stored streams and what is still pending.
        rows: only these rows of the batch."""
        r = self.reads[q]
        if rows is not None:
            x, pending = x[rows], [(y[rows], s) for y, s in pending]
        x, h = ops.mix_streams(x, pending, r.coef, r.rewrite, norm, eps, dtype)
        return h, x, [] if r.rewrite else pending
