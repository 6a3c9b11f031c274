"""Mixture-of-experts ops: routing, the experts' grouped products, and the
pending sum over a token's experts (ops/csrc/experts.hip on the GPU,
ops/reference_hybrid.py on the CPU)."""

from __future__ import annotations

from dataclasses import dataclass
from typing import Callable, Optional, Tuple

import torch

from . import reference_hybrid as ref
from .native import hybrid_native


@dataclass
class ExpertWeights:
    """gate_up and down of all experts: in MFMA fragments [E, N/16, K/32, 64,
    8] (gate and up rows alternate in blocks of 16), or dense [E, 2 ff, W] and
    [E, W, ff]."""

    gate_up: torch.Tensor
    down: torch.Tensor
    ff: int
    width: int
    experts: int

    @property
    def fragments(self) -> bool:
        return self.gate_up.dim() == 5


@dataclass
class Routing:
    """Where a token's choices went: slot [T, top] is the row, in the order by
    expert, of its j-th expert; weights [T, top] fp32."""

    slot: torch.Tensor
    weights: torch.Tensor
    ids: torch.Tensor                            # [T, top] int32
    row_token: Optional[torch.Tensor] = None     # [rows] int32, -1: no row (GPU)
    tile_info: Optional[torch.Tensor] = None     # [4 * tiles + 1] int32, see experts.hip
    tile_rows: int = 0


@dataclass
class ExpertSum:
    """sum_j weights[t, j] * rows[slot[t, j]] (+ shared[t]), not added up yet:
    the stream kernel does it."""

    rows: torch.Tensor
    slot: torch.Tensor
    weights: torch.Tensor
    shared: Optional[torch.Tensor]

    def __getitem__(self, idx) -> "ExpertSum":
        shared = None if self.shared is None else self.shared[idx]
        return ExpertSum(self.rows, self.slot[idx], self.weights[idx], shared)

    def float(self) -> torch.Tensor:
        return ref.expert_sum(self.rows, self.slot, self.weights, self.shared)


def _fragments(w: torch.Tensor) -> torch.Tensor:
    """[N, K] (zero-padded to multiples of 256 and 64) -> [N/16, K/32, 64, 8]:
    lane l of a fragment holds W[l % 16][8 (l / 16) ..]."""
    N, K = w.shape
    w = torch.nn.functional.pad(w, (0, -K % 64, 0, -N % 256))
    w = w.view(w.shape[0] // 16, 16, w.shape[1] // 32, 4, 8)
    return w.permute(0, 2, 3, 1, 4).reshape(w.shape[0], w.shape[2], 64, 8)


def _interleave(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    """Blocks of 16 gate rows and 16 up rows in turn."""
    pad = (0, 0, 0, -gate.shape[0] % 16)
    g, u = (torch.nn.functional.pad(w, pad).view(-1, 16, w.shape[1]) for w in (gate, up))
    return torch.stack([g, u], 1).view(-1, gate.shape[1])


def pack_experts(
    ff: int, width: int, experts: int, get: Callable[[int], Tuple[torch.Tensor, ...]]
) -> ExpertWeights:
    """get(e): the (gate, up, down) of an expert; one is held at a time."""
    gate_up = down = None
    for e in range(experts):
        g, u, d = get(e)
        if g.is_cuda and g.dtype == torch.bfloat16 and ff % 8 == 0 and width % 8 == 0:
            a, b = _fragments(_interleave(g, u)), _fragments(d)
        else:
            a, b = torch.cat([g, u]), d
        if gate_up is None:
            gate_up, down = a.new_empty(experts, *a.shape), b.new_empty(experts, *b.shape)
        gate_up[e], down[e] = a, b
    return ExpertWeights(gate_up, down, ff, width, experts)


def _tile_rows(choices: int, w: ExpertWeights) -> int:
    """Rows per tile: what a tile of an average expert needs."""
    if not w.fragments:
        return 16
    mean = choices / w.experts
    return 16 if mean <= 10 else 32 if mean <= 20 else 64 if mean <= 48 else 256


def route_experts(
    h, w_router, bias, top: int, experts: ExpertWeights, scale: float = 1.0
) -> Routing:
    """The ``top`` experts of every row by logits h w_router^T (+ bias; fp32),
    weighted by ``scale`` times the softmax over the chosen logits."""
    from .hybrid import linear_f32

    z = linear_f32(h, w_router)
    if not h.is_cuda:
        ids, weights = ref.route_experts(z if bias is None else z + bias, top)
        weights *= scale
        slot = torch.arange(ids.numel(), dtype=torch.int32).view(ids.shape)
        return Routing(slot, weights, ids.int())
    T, dev = h.shape[0], h.device
    n = T * top
    rows = _tile_rows(n, experts)
    tiles = min(n, experts.experts + n // rows)
    sizes = (4 * tiles + 1, n, n, tiles * rows)
    ints = torch.empty(sum(sizes), dtype=torch.int32, device=dev)
    tile_info, ids, slot, row_token = ints.split(sizes)
    ids, slot = ids.view(T, top), slot.view(T, top)
    weights = torch.empty(T, top, dtype=torch.float32, device=dev)
    hybrid_native().route(ids, weights, slot, row_token, tile_info, z, bias, scale, rows)
    return Routing(slot, weights, ids, row_token, tile_info, rows)


def expert_rows(
    h, routing: Routing, w: ExpertWeights, limit: Optional[float]
) -> torch.Tensor:
    """The chosen experts' outputs, a row each at routing.slot; ``limit``: of
    the clamped GLU, None for silu(gate) * up."""
    if not h.is_cuda:
        return ref.expert_rows(h, routing.ids, w.gate_up, w.down, limit)
    R, ext = routing.row_token.numel(), hybrid_native()
    act = torch.empty(R, w.ff, dtype=h.dtype, device=h.device)
    out = torch.empty(R, w.width, dtype=h.dtype, device=h.device)
    where = (routing.row_token, routing.tile_info, routing.tile_rows)
    ext.expert_product(
        act, h, w.gate_up, *where, 2 if limit is None else 1, float(limit or 0.0)
    )
    ext.expert_product(out, act, w.down, *where, 0, 0.0)
    return out


def clamped_glu(x: torch.Tensor, limit: float) -> torch.Tensor:
    """g sigmoid(1.702 g) (u + 1) of x = [gate | up], g clamped from above and
    u on both sides."""
    if not x.is_cuda:
        return ref.clamped_glu(x, limit)
    out = torch.empty(x.shape[0], x.shape[1] // 2, dtype=x.dtype, device=x.device)
    hybrid_native().clamped_glu(out, x, float(limit))
    return out
