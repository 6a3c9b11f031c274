"""Ops of the hybrid decoders: gfx950 kernels (the ``_H`` extension) on GPU
tensors, ops/reference_hybrid.py on CPU tensors.

Rows are those of a flat batch; ``segs`` (models/batch.py Segments) says
which sequence each belongs to, where its pages and state are. Every op
takes any split of a sequence into segments.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, Optional, Sequence, Tuple

import numpy as np
import torch

from . import reference_hybrid as ref
from .native import hybrid_native
from .reference_hybrid import build_pair_rope_cache


# ---------------------------------------------------------------- planning
@dataclass
class Unfold:
    """Prefill rows [0, rows) attend through per-head keys and values made
    from ``keys`` latents, gathered from the pages sequence by sequence."""

    rows: int
    keys: int
    key_slots: torch.Tensor   # [keys] int64 global cache rows
    cu_q: torch.Tensor        # [S+1] int32
    cu_k: torch.Tensor        # [S+1] int32
    tile_seg: torch.Tensor    # [ntiles] int32
    tile_off: torch.Tensor    # [ntiles] int32
    tile_rows: int            # query rows per tile


@dataclass
class Chunks:
    """Segments long enough for the chunked form of the recurrences."""

    # int32: the segments, the first chunk of each (and the end), then per
    # chunk its segment and its first row within it
    maps: Tuple[torch.Tensor, torch.Tensor, torch.Tensor, torch.Tensor]
    short: Optional[torch.Tensor]  # int32 segments that run token by token


@dataclass
class Tiles:
    """Segments long enough for the tiled form of paged attention."""

    tile_seg: torch.Tensor          # [ntiles] int32
    tile_off: torch.Tensor          # [ntiles] int32 first row within the segment
    tile_rows: int
    rest: Optional[torch.Tensor]    # int32 rows of the other segments


@dataclass
class SegmentPlan:
    """How a step's rows go through the kernels; made once per step.
    ``carry``: rows that one layer leaves for later layers of the step."""

    unfold: Optional[Unfold] = None
    chunks: Optional[Chunks] = None
    tiles: Optional[Tiles] = None
    head_tiles: Optional[Tiles] = None
    carry: Dict[str, torch.Tensor] = field(default_factory=dict)


CHUNK = 64            # rows per chunk of the chunked recurrences
CHUNK_MIN_ROWS = 32   # shorter segments run token by token
UNFOLD_RATIO = 16     # query-key pairs per key from which unfolding pays
TILE_MIN_ROWS = 16    # shorter segments attend row by row
HEAD_TILE = 16        # query rows per tile where a tile holds all heads
PLANS = ("unfold", "chunks", "tiles", "head_tiles")


def plan_segments(batch, dtype, parts_of=PLANS) -> SegmentPlan:
    """parts_of: the parts that the model's mixers use."""
    segs = batch.segs
    plan = SegmentPlan()
    if batch.kind == "decode" or segs.lens is None:
        return plan
    if not batch.token_ids.is_cuda or dtype != torch.bfloat16:
        return plan
    dev = batch.token_ids.device
    lens, starts = segs.lens, segs.starts
    nseg_p = segs.n_prefill
    parts, fields = [], []

    def put(name, a):
        fields.append((name, len(a)))
        parts.append(np.asarray(a, dtype=np.int32))

    pl, ps = lens[:nseg_p], starts[:nseg_p]
    keys = int((pl + ps).sum())
    pairs = float((pl * (ps + pl / 2.0)).sum())
    unfold = "unfold" in parts_of and nseg_p > 0 and pairs >= UNFOLD_RATIO * keys
    tiled = np.nonzero(lens >= TILE_MIN_ROWS)[0]
    kinds = {}  # name of the tiled form -> rows per tile
    if len(tiled):
        if "tiles" in parts_of:
            kinds["tiles"] = 128 if int(lens[tiled].max()) > 64 else 64
        if "head_tiles" in parts_of:
            kinds["head_tiles"] = HEAD_TILE
    if unfold:
        put("cu_q", np.concatenate([[0], np.cumsum(pl)]))
        put("cu_k", np.concatenate([[0], np.cumsum(pl + ps)]))
        tile_rows = 128 if int(pl.max()) > 64 else 64
        seg = np.repeat(np.arange(nseg_p), -(-pl // tile_rows))
        off = np.concatenate([np.arange(0, n, tile_rows) for n in pl])
        order = np.argsort(-(ps[seg] + off), kind="stable")  # longest first
        put("tile_seg", seg[order])
        put("tile_off", off[order])
    for name, rows_t in kinds.items():
        n = lens[tiled]
        seg = np.repeat(tiled, -(-n // rows_t))
        off = np.concatenate([np.arange(0, k, rows_t) for k in n])
        if name == "tiles":
            order = np.argsort(-(starts[seg] + off), kind="stable")  # longest first
            seg, off = seg[order], off[order]
        put(name + "_seg", seg)
        put(name + "_off", off)
    if kinds:
        put("tile_rest", np.nonzero(np.repeat(lens < TILE_MIN_ROWS, lens))[0])
    long = np.nonzero(lens >= CHUNK_MIN_ROWS)[0] if "chunks" in parts_of else np.empty(0, int)
    nchunk = (lens[long] + CHUNK - 1) // CHUNK
    if len(long):
        put("segs", long)
        put("first", np.concatenate([[0], np.cumsum(nchunk)]))
        put("chunk_seg", np.repeat(long, nchunk))
        put("chunk_off", np.concatenate([np.arange(n) * CHUNK for n in nchunk]))
        put("short", np.nonzero(lens < CHUNK_MIN_ROWS)[0])
    if not parts:
        return plan
    flat = torch.from_numpy(np.concatenate(parts)).to(dev)  # one copy for all maps
    got, at = {}, 0
    for name, n in fields:
        got[name] = flat[at : at + n]
        at += n
    if unfold:
        tables = segs.tables[:nseg_p]
        cu_k = got["cu_k"].long()
        seg = torch.repeat_interleave(
            torch.arange(nseg_p, device=dev), cu_k.diff(), output_size=keys
        )
        pos = torch.arange(keys, device=dev) - cu_k[seg]
        bs = segs.block_size
        plan.unfold = Unfold(
            rows=batch.n_prefill_tokens, keys=keys,
            key_slots=tables[seg, pos // bs].long() * bs + pos % bs,
            cu_q=got["cu_q"], cu_k=got["cu_k"],
            tile_seg=got["tile_seg"], tile_off=got["tile_off"],
            tile_rows=tile_rows,
        )
    for name, rows_t in kinds.items():
        setattr(plan, name, Tiles(
            tile_seg=got[name + "_seg"], tile_off=got[name + "_off"], tile_rows=rows_t,
            rest=got["tile_rest"] if got["tile_rest"].numel() else None,
        ))
    if len(long):
        plan.chunks = Chunks(
            maps=tuple(got[k] for k in ("segs", "first", "chunk_seg", "chunk_off")),
            short=got["short"] if got["short"].numel() else None,
        )
    return plan


# ------------------------------------------------------ stream and products
def linear_f32(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x @ w.T with the fp32 accumulator as the result."""
    if x.dtype == torch.float32:
        return torch.nn.functional.linear(x, w)
    if x.is_cuda:
        return torch.mm(x, w.t(), out_dtype=torch.float32)
    return torch.nn.functional.linear(x.float(), w.float())


def embed_scaled(tokens, embed, scale: float, x0: Optional[torch.Tensor]) -> torch.Tensor:
    """fp32 embed[token] * scale; x0 (compute dtype, may be strided)
    receives the same rows."""
    if not embed.is_cuda:
        return ref.embed_scaled(tokens, embed, scale, x0)
    x = torch.empty(tokens.shape[0], embed.shape[1], dtype=torch.float32, device=embed.device)
    hybrid_native().embed_scaled(x, x0, tokens, embed, float(scale))
    return x


def add_layernorm(x, delta, w, b, eps: float, dtype, vec=None, replace: bool = False):
    """x (fp32 stream, in place) += delta [+ vec], or = delta [+ vec] with
    ``replace``; returns layer norm(x) * w + b in ``dtype``."""
    if not x.is_cuda:
        return ref.add_layernorm(x, delta, w, b, eps, dtype, vec, replace)
    out = torch.empty(x.shape, dtype=dtype, device=x.device)
    hybrid_native().add_layernorm(out, x, delta, vec, w, b, float(eps), replace)
    return out


def add_rms_norm(x, deltas: Sequence, weights: Sequence[torch.Tensor], eps: float, dtype):
    """x (fp32 stream, in place) += every one of deltas: at most one tensor
    and one ExpertSum, or two tensors; returns, for each of one or two norm
    weights, RMS norm(x) * weight in ``dtype``."""
    if not x.is_cuda:
        return ref.add_rms_norm(x, deltas, weights, eps, dtype)
    outs = tuple(torch.empty(x.shape, dtype=dtype, device=x.device) for _ in weights)
    parts = [d for d in deltas if not isinstance(d, ExpertSum)]
    sums = [d for d in deltas if isinstance(d, ExpertSum)]
    assert len(outs) in (1, 2) and len(parts) <= 2 and len(sums) <= (1 if len(parts) < 2 else 0)
    e = sums[0] if sums else None
    if e is not None and e.shared is not None:
        raise NotImplementedError("RMS norm after experts with a shared one")
    hybrid_native().add_rms_norm(
        outs[0], outs[1] if len(outs) > 1 else None, x, *(parts + [None, None])[:2],
        *((e.rows, e.slot, e.weights) if e is not None else (None, None, None)),
        weights[0], weights[1] if len(outs) > 1 else None, float(eps),
    )
    return outs


def add_cast(x, delta, out) -> None:
    """x += delta; out (compute dtype, may be strided) = x."""
    if not x.is_cuda:
        return ref.add_cast(x, delta, out)
    hybrid_native().add_cast(out, x, delta)


def head_linear(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """y[t, h] = w[h] @ x[t, h]: x [T, H, K], w [H, N, K]."""
    if not x.is_cuda:
        return ref.head_linear(x, w)
    y = torch.empty(x.shape[0], w.shape[0], w.shape[1], dtype=x.dtype, device=x.device)
    hybrid_native().head_linear(y, x, w)
    return y


# ---------------------------------------------------------- latent attention
def latent_rows(d, q_norm, kv_norm, eps, rot, positions, cos_sin, latent, slot_mapping):
    """d [T, q_rank + kv_rank + rot]: returns the normed query latent; writes
    [normed kv latent | rotated key part] into the paged cache."""
    if not d.is_cuda:
        return ref.latent_rows(
            d, q_norm, kv_norm, eps, rot, positions, cos_sin, latent, slot_mapping
        )
    cq = torch.empty(d.shape[0], q_norm.numel(), dtype=d.dtype, device=d.device)
    hybrid_native().latent_rows(
        cq, latent, d, q_norm, kv_norm, float(eps), rot, positions, cos_sin, slot_mapping
    )
    return cq


def fold_queries(q, uk_t, row: int, cos_sin, positions) -> torch.Tensor:
    """[T, H, row]: W_uk^T q_unrotated, the rotated part, zeros up to row."""
    if not q.is_cuda:
        return ref.fold_queries(q, uk_t, row, positions, cos_sin)
    H, rank, dim = uk_t.shape
    out = torch.empty(q.shape[0], H, row, dtype=q.dtype, device=q.device)
    hybrid_native().head_linear(out[..., :rank], q[..., :dim], uk_t)
    hybrid_native().rotate_pairs(out[..., rank:], q[..., dim:], positions, cos_sin)
    return out


def latent_attention_folded(ql, latent, rank, sink, scale, positions, segs, row0: int):
    """Row t (row row0 + t of the flat batch) against its sequence's cached
    rows 0..positions[t]; returns the latent-space sums [T, H, rank]."""
    if not ql.is_cuda:
        return ref.latent_attention_folded(
            ql, latent, rank, sink, scale, positions, segs, row0
        )
    T, H, row = ql.shape
    out = torch.empty(T, H, rank, dtype=ql.dtype, device=ql.device)
    nsplit, pa, pm = 0, None, None
    page = latent.shape[1]
    if ql.dtype == torch.bfloat16 and row <= 576 and page & (page - 1) == 0:
        # fill the chip: splits only from shapes, so captured graphs hold
        max_tiles = -(-segs.tables.shape[1] * page // 64)
        nsplit = max(1, min(-(-256 // (T * -(-H // 32))), 16, max_tiles))
        if nsplit > 1:
            pa, pm = _folded_scratch(ql.device, T * H * nsplit * rank, T * H * nsplit * 2)
    hybrid_native().latent_attention_folded(
        out, ql, latent, sink, float(scale), positions, segs.row_seg[row0:], segs.tables,
        nsplit, pa, pm,
    )
    return out


_scratch: dict = {}
_scratch_retired: list = []


def _folded_scratch(device, n_acc: int, n_ml: int):
    """fp32 scratch shared by all launches of a device (stream order)."""
    ws = _scratch.get(device.index)
    if ws is None or ws[0].numel() < n_acc or ws[1].numel() < n_ml:
        if ws is not None:
            _scratch_retired.append(ws)  # captured graphs may still use it
            n_acc, n_ml = max(n_acc, ws[0].numel()), max(n_ml, ws[1].numel())
        ws = (
            torch.empty(n_acc, dtype=torch.float32, device=device),
            torch.empty(n_ml, dtype=torch.float32, device=device),
        )
        _scratch[device.index] = ws
    return ws


def can_unfold(dim: int, rot: int, vdim: int, rank: int) -> bool:
    """Whether latent_attention_unfolded has a kernel for these sizes."""
    return (
        all(d % 8 == 0 for d in (dim, rot, vdim, rank)) and dim + rot <= 256 and vdim <= 256
    )


def latent_attention_unfolded(q, latent, w_ukv, sink, scale, dim, vdim, rank, cos_sin,
                              positions, u: Unfold) -> torch.Tensor:
    """Rows [0, u.rows) of q [T, H, dim + rot] (rotated in place) against
    keys and values unfolded from their sequences' latents by w_ukv
    [H*dim | H*vdim, rank]; returns [T, H, vdim], later rows unset. bf16 on
    the GPU only: the folded form is the same function."""
    T, H = q.shape[0], q.shape[1]
    ext = hybrid_native()
    ext.rotate_pairs(
        q[: u.rows, :, dim:], q[: u.rows, :, dim:], positions[: u.rows], cos_sin
    )
    lat = latent.view(-1, latent.shape[-1])[u.key_slots]
    kv = torch.nn.functional.linear(lat[:, :rank], w_ukv)
    out = torch.empty(T, H, vdim, dtype=q.dtype, device=q.device)
    ext.latent_attention_unfolded(
        out, q, kv, lat, sink, float(scale), u.cu_q, u.cu_k, u.tile_seg, u.tile_off,
        u.tile_rows, dim, vdim, rank,
    )
    return out


# --------------------------------------------------------------- recurrences
def causal_conv(x, w_t, b, state, positions, segs, plan) -> torch.Tensor:
    """silu of the causal per-channel convolution of x [T, C] (may be
    strided) with taps w_t [taps, C]; state [slots, taps-1, C] carries the last inputs."""
    if not x.is_cuda:
        return ref.causal_conv(x, w_t, b, state, positions, segs)
    y = torch.empty(x.shape, dtype=x.dtype, device=x.device)
    hybrid_native().causal_conv(
        y, x, w_t, b, state, positions, segs.cu, segs.slots, segs.row_seg
    )
    return y


def ssd(xbc, dt, dt_bias, A_log, D, H, P, N, G, S, positions, segs, plan):
    """Mamba-2 recurrence over xbc [T, H*P + 2*G*N] and raw dt [T, H]
    (fp32); state S [slots, H, P, N]."""
    if not xbc.is_cuda:
        return ref.ssd(xbc, dt, dt_bias, A_log, D, H, P, N, G, S, positions, segs)
    y = torch.empty(xbc.shape[0], H * P, dtype=xbc.dtype, device=xbc.device)
    ext, ch = hybrid_native(), plan.chunks
    args = (y, xbc, dt, dt_bias, A_log, D, H, P, N, G, S, positions, segs.cu, segs.slots)
    if ch is not None and P % 8 == 0 and N % 8 == 0:
        ext.ssd_chunked(*args, *ch.maps)
        if ch.short is not None:
            ext.ssd_scan(*args, ch.short)
    else:
        ext.ssd_scan(*args, None)
    return y


def mlstm(q, k, v, gates, bias, cap, H, dk, dv, S, n, m, positions, segs, plan):
    """mLSTM recurrence; gates [T, 2H] fp32 raw input and forget gates,
    states S [slots, H, dv, dk], n [slots, tiles, H, dk], m [slots, tiles, H]
    (a copy per tile of 64 value rows)."""
    if not q.is_cuda:
        return ref.mlstm(q, k, v, gates, bias, cap, H, dk, dv, S, n, m, positions, segs)
    y = torch.empty(q.shape[0], H * dv, dtype=q.dtype, device=q.device)
    ext, ch = hybrid_native(), plan.chunks
    args = (y, q, k, v, gates, bias, float(cap), H, dk, dv, S, n, m, positions, segs.cu,
            segs.slots)
    if ch is not None and dk % 8 == 0 and dv % 8 == 0:
        ext.mlstm_chunked(*args, *ch.maps)
        if ch.short is not None:
            ext.mlstm_scan(*args, ch.short)
    else:
        ext.mlstm_scan(*args, None)
    return y


def gated_norm(y, gate, w, groups: int, eps: float, gate_first: bool):
    """RMS norm of y in ``groups`` equal parts, times w; multiplied by
    silu(gate) before the norm, or by sigmoid(gate) after it."""
    if not y.is_cuda:
        return ref.gated_norm(y, gate, w, groups, eps, gate_first)
    out = torch.empty_like(y)
    hybrid_native().gated_norm(out, y, gate, w, groups, float(eps), 1 if gate_first else 0)
    return out


def head_norm_gate(out, y, gate, w, heads: int, eps: float, act: str = "silu") -> None:
    """out = RMS norm of y per head, times w, times silu(gate) (act "sigmoid":
    sigmoid(gate)); out and gate may be strided."""
    if not y.is_cuda:
        return ref.head_norm_gate(out, y, gate, w, heads, eps, act)
    hybrid_native().head_norm_gate(out, y, gate, w, heads, float(eps), act == "sigmoid")


# ------------------------------------------------------------- dynamic tanh
def add_tanh_norm(x, delta, post, norm, dtype, replace: bool = False, out=None):
    """x (fp32 stream, in place) += post(delta), or = with ``replace``;
    returns norm(x), or x without a norm, in ``dtype`` (written to ``out`` if
    given, which may be strided). Norms are (w, b, alpha):
    tanh(alpha z) * w + b. delta: None, a tensor, or an ExpertSum."""
    if not x.is_cuda:
        return ref.add_tanh_norm(x, delta, post, norm, dtype, replace, out)
    if out is None:
        out = torch.empty(x.shape, dtype=dtype, device=x.device)
    parts = (delta, None, None, None, None)
    if isinstance(delta, ExpertSum):
        parts = (None, delta.rows, delta.slot, delta.weights, delta.shared)
    none = (None, None, 1.0)
    hybrid_native().stream_tanh(out, x, *parts, *(post or none), *(norm or none), replace)
    return out


def embed_tanh_norm(tokens, embed, norm, x0: Optional[torch.Tensor]) -> torch.Tensor:
    """fp32 norm(embed[token]); x0 as in embed_scaled."""
    if not embed.is_cuda:
        return ref.embed_tanh_norm(tokens, embed, norm, x0)
    x = torch.empty(tokens.shape[0], embed.shape[1], dtype=torch.float32, device=embed.device)
    hybrid_native().embed_tanh(x, x0, tokens, embed, *norm)
    return x


def soft_cap_(x: torch.Tensor, cap: float) -> None:
    """x (fp32) = cap * tanh(x / cap) in place."""
    if not x.is_cuda:
        return ref.soft_cap_(x, cap)
    hybrid_native().soft_cap(x, float(cap))


# ------------------------------------------------- attention over k/v pages
def page_write(k, v, k_pages, v_pages, slot_mapping) -> None:
    """Rows of keys and values (may be strided) into their cache slots."""
    if not k.is_cuda:
        return ref.page_write(k, v, k_pages, v_pages, slot_mapping)
    hybrid_native().page_write(k, v, k_pages, v_pages, slot_mapping)


def paged_attention(out, q, k_pages, v_pages, H: int, G: int, sink, scale: float, cap: float,
                    gate, out_scale: float, positions, segs, plan: SegmentPlan) -> None:
    """Causal attention of every row to its sequence's pages (its own token
    among them): scores cap*tanh(scale q.k/cap), a sink per head in the
    denominator; out [T, H*vdim] is multiplied by sigmoid(gate [T, H]) and
    out_scale. q, gate and out may be strided."""
    if not q.is_cuda:
        return ref.paged_attention(
            out, q, k_pages, v_pages, H, G, sink, scale, cap, gate, out_scale, positions, segs
        )
    ext = hybrid_native()
    page, dim, vdim = k_pages.shape[1], k_pages.shape[2] // G, v_pages.shape[2] // G
    head = (out, q, k_pages, v_pages, H, G, sink, float(scale), float(cap), gate,
            float(out_scale), positions)
    mfma = (
        q.dtype == torch.bfloat16 and page >= 16 and page & (page - 1) == 0
        and dim % 8 == 0 and vdim % 8 == 0 and dim <= 256 and vdim <= 256
    )
    rows, n = None, q.shape[0]
    if mfma and plan.tiles is not None:
        t = plan.tiles
        ext.paged_tiles(
            *head, segs.tables, segs.cu, t.tile_seg, t.tile_off, t.tile_rows
        )
        if t.rest is None:
            return
        rows, n = t.rest, t.rest.numel()
    nsplit, pa, pm = 0, None, None
    if mfma:
        # fill the chip: splits only from shapes, so captured graphs hold
        groups = n * G * -(-(H // G) // 16)
        max_tiles = -(-segs.tables.shape[1] * page // 128)
        nsplit = max(1, min(-(-512 // groups), 16, max_tiles))
        if nsplit > 1:
            pa, pm = _folded_scratch(q.device, n * H * nsplit * vdim, n * H * nsplit * 2)
    ext.paged_rows(*head, segs.row_seg, segs.tables, rows, nsplit, pa, pm)


# ------------------------------- sigmoid attention over pages, mixed heads
def distance_bias(rel: torch.Tensor, pb: torch.Tensor, bias_max: float, window: int):
    """fp32 [distances, heads padded to 16]: rel[bucket(n), h] + pb[h] for
    distances n = 0, 1, ...; the last row also serves all larger ones. rel
    [B, H] has a row per distance below B/2, then rows of logarithmically
    growing width up to distance bias_max, beyond which all share the last."""
    B, H = rel.shape
    half = B // 2
    last = min(int(np.ceil(bias_max)), window - 1)
    n = np.arange(last + 1)
    # (the nudge: where the logarithms' ratio is an integer, rounding must
    # not take the floor below it)
    log = np.log(np.maximum(n, half) / half) / np.log(bias_max / half) * (B - half) + 1e-9
    row = np.where(n < half, n, np.minimum(B - 1, half + np.floor(log).astype(np.int64)))
    out = torch.zeros(last + 1, -(-H // 16) * 16, dtype=torch.float32, device=rel.device)
    out[:, :H] = rel.float()[torch.from_numpy(row).to(rel.device)] + pb.float()
    return out


def qkv_rows(q, k, v, q_norm, k_norm, eps: float, blend: float, v_first, k_pages, v_pages,
             slot_mapping) -> torch.Tensor:
    """RMS norm over a whole row of q (returned) and of k; keys and values,
    blended to (1 - blend) v + blend v_first where v_first is given, go to
    their cache slots. q, k, v, v_first may be strided."""
    if not q.is_cuda:
        return ref.qkv_rows(q, k, v, q_norm, k_norm, eps, blend, v_first, k_pages, v_pages,
                            slot_mapping)
    out = torch.empty(q.shape, dtype=q.dtype, device=q.device)
    hybrid_native().qkv_rows(
        out, q, k, v, q_norm, k_norm, float(eps), float(blend), v_first, k_pages, v_pages,
        slot_mapping,
    )
    return out


def sigmoid_attention(out, q, k_pages, v_pages, H: int, G: int, scale: float, bias, talk,
                      window: int, gate, positions, segs, plan: SegmentPlan) -> None:
    """Every row's attention to the last ``window`` rows of its sequence's
    pages (its own token among them). Weights sigmoid(scale q.k +
    bias[distance]) (bias: distance_bias) are not normalized; head h takes
    sum_g talk[h, g] of all heads' weights to the values of its key head. out
    [T, H*vdim] is multiplied by sigmoid(gate) element by element. q, gate
    and out may be strided."""
    if not q.is_cuda:
        return ref.sigmoid_attention(
            out, q, k_pages, v_pages, H, G, scale, bias, talk, window, gate, positions, segs
        )
    ext = hybrid_native()
    page, dim, vdim = k_pages.shape[1], k_pages.shape[2] // G, v_pages.shape[2] // G
    head = (out, q, k_pages, v_pages, H, G, float(scale), bias, talk, int(window), gate,
            positions)
    most = 256 if H <= 32 else 128
    mfma = (
        q.dtype == torch.bfloat16 and page >= 16 and page & (page - 1) == 0 and H <= 64
        and dim % 8 == 0 and vdim % 8 == 0 and dim <= most and vdim <= most
    )
    rows, n = None, q.shape[0]
    per_wave = -(-H // 8)  # a tile's 8 waves share the heads, no wave has two key heads
    if (
        mfma and plan.head_tiles is not None and per_wave <= 4 and H // G % per_wave == 0
        and dim <= 128 and vdim <= 128
    ):
        t = plan.head_tiles
        ext.sigmoid_tiles(*head, segs.tables, segs.cu, t.tile_seg, t.tile_off)
        if t.rest is None:
            return
        rows, n = t.rest, t.rest.numel()
    nsplit, part = 0, None
    if mfma:
        # fill the chip: splits only from shapes, so captured graphs hold
        most = -(-min(segs.tables.shape[1] * page, window + 31) // 128)
        nsplit = max(1, min(-(-256 // n), 16, most))
        if nsplit > 1:
            part, _ = _folded_scratch(q.device, n * H * nsplit * vdim, 0)
    ext.sigmoid_rows(*head, segs.row_seg, segs.tables, rows, nsplit, part)


# -------------------------------------- recurrences with a decay per channel
DECAY_KINDS = {"sigmoid": 0, "exp": 1, "softplus": 2}


def decay_logs(a, w2, bias, kind: str, tau: float = 1.0, rate=None) -> torch.Tensor:
    """fp32 log decays [T, N] from a [T, rank] (may be strided), with
    z = a w2^T + bias: "sigmoid": log sigmoid(z) / tau; "softplus":
    -rate * softplus(z), rate [N]; "exp": -e^z of z = tanh(a) w2^T + bias."""
    if not a.is_cuda:
        return ref.decay_logs(a, w2, bias, kind, tau, rate)
    out = torch.empty(a.shape[0], w2.shape[0], dtype=torch.float32, device=a.device)
    hybrid_native().decay_logs(out, a, w2, bias, DECAY_KINDS[kind], float(tau), rate)
    return out


def token_shift(h, mu, prev, positions, segs) -> torch.Tensor:
    """[mixes, T, W]: h + (h' - h) * mu[m] with h' the sequence's previous
    row (zeros before the first); prev [slots, W] carries each sequence's
    last row."""
    if not h.is_cuda:
        return ref.token_shift(h, mu, prev, positions, segs)
    out = torch.empty(mu.shape[0], *h.shape, dtype=h.dtype, device=h.device)
    hybrid_native().token_shift(out, h, mu, prev, positions, segs.cu, segs.slots, segs.row_seg)
    return out


def decayed_kv(q, k, v, logw, u, qscale: float, H: int, dk: int, dv: int, S, positions, segs,
               plan: SegmentPlan) -> torch.Tensor:
    """S = diag(e^logw) S + k v^T per head, read out by q: after the update
    (u None), or before it with a bonus u for the current token. q, k, v may
    be strided; logw [T, H*dk] fp32 is consumed; S [slots, H, dv, dk]."""
    if not q.is_cuda:
        return ref.decayed_kv(q, k, v, logw, u, qscale, H, dk, dv, S, positions, segs)
    y = torch.empty(q.shape[0], H * dv, dtype=q.dtype, device=q.device)
    ext, ch = hybrid_native(), plan.chunks
    args = (y, q, k, v, logw, u, float(qscale), H, dk, dv, S, positions, segs.cu, segs.slots)
    if ch is not None and dk % 8 == 0 and dv % 8 == 0 and dk <= 256:
        if ch.short is not None:
            ext.decay_scan(*args, ch.short)
        ext.decay_chunked(*args, *ch.maps)
    else:
        ext.decay_scan(*args, None)
    return y


# --------------------------------------------------- hyper-connected streams
def embed_rms_norm(tokens, embed, w, eps: float) -> torch.Tensor:
    """fp32 RMS norm(embed[token]) * w."""
    if not embed.is_cuda:
        return ref.embed_rms_norm(tokens, embed, w, eps)
    x = torch.empty(tokens.shape[0], embed.shape[1], dtype=torch.float32, device=embed.device)
    hybrid_native().embed_rms_norm(x, tokens, embed, w, float(eps))
    return x


def mix_streams(x, pending, coef, rewrite: bool, w, eps: float, dtype):
    """Linear combinations of the rows x[:, s] (fp32 [T, streams, W]) and of
    the pending sublayer outputs, (y [T, W], scale [W] or None) each: coef
    [streams + pending, columns]. Returns (streams, RMS norm of the first
    column's * w in ``dtype``); the streams are the other columns with
    ``rewrite`` (in x's memory where it fits), x as it is without."""
    if not x.is_cuda:
        return ref.mix_streams(x, pending, coef, rewrite, w, eps, dtype)
    T, S, W = x.shape
    out = x
    if rewrite and coef.shape[1] - 1 != S:
        out = torch.empty(T, coef.shape[1] - 1, W, dtype=torch.float32, device=x.device)
    h = torch.empty(T, W, dtype=dtype, device=x.device)
    ys, scales = [y for y, _ in pending], [s for _, s in pending]
    hybrid_native().mix_streams(h, out if rewrite else None, x, ys, scales, coef, w, float(eps))
    return out, h


def xielu_(z: torch.Tensor, pos: float, neg: float) -> torch.Tensor:
    """z = pos z^2 + z/2 where z > 0, neg (e^z - 1 - z) + z/2 else, in place."""
    if not z.is_cuda:
        return ref.xielu_(z, pos, neg)
    hybrid_native().xielu(z, float(pos), float(neg))
    return z


# ------------------------ rotary attention in a window, differential or plain
def rotary_rows(q, k, v, q_norm, k_norm, eps: float, cos_sin, positions, k_pages, v_pages,
                slot_mapping) -> torch.Tensor:
    """RMS norm of every dim = q_norm.numel() values of q (returned) and k,
    then the rotation of the first cos_sin.shape[1] of them in halves; keys
    and values go to their cache slots (k None: another layer wrote them).
    q, k, v may be strided."""
    if not q.is_cuda:
        return ref.rotary_rows(q, k, v, q_norm, k_norm, eps, cos_sin, positions, k_pages,
                               v_pages, slot_mapping)
    out = torch.empty(q.shape, dtype=q.dtype, device=q.device)
    hybrid_native().rotary_rows(
        out, q, k, v, q_norm, k_norm, float(eps), cos_sin, positions,
        *((k_pages, v_pages, slot_mapping) if k is not None else (None, None, None)),
    )
    return out


def window_attention(out, q, k_pages, v_pages, H: int, G: int, maps: int, scale: float,
                     window: int, keep_first: int, lam: float, gain: float, eps: float,
                     positions, segs, plan: SegmentPlan) -> None:
    """Softmax attention of every row to its sequence's pages: a row at
    position p sees j <= p with p - j < window or j < keep_first. A head has
    ``maps`` (1 or 2) queries, a key head as many keys, all over the same
    values: with one, out is its output; with two, a1 and a2, it is the RMS
    norm of a1 - lam a2 over the head, times gain. q and out [T, H*vdim] may
    be strided."""
    window, keep_first = min(int(window), 1 << 30), min(int(keep_first), 1 << 30)
    if not q.is_cuda:
        return ref.window_attention(
            out, q, k_pages, v_pages, H, G, maps, scale, window, keep_first, lam, gain, eps,
            positions, segs,
        )
    ext = hybrid_native()
    page = k_pages.shape[1]
    dim, vdim = k_pages.shape[2] // (G * maps), v_pages.shape[2] // G
    head = (out, q, k_pages, v_pages, H, G, maps, float(scale), window, keep_first, float(lam),
            float(gain), float(eps), positions)
    mfma = (
        q.dtype == torch.bfloat16 and page >= 16 and page & (page - 1) == 0
        and dim % 8 == 0 and vdim % 8 == 0 and dim * maps <= 256 and vdim <= 256
    )
    rows, n = None, q.shape[0]
    if mfma and plan.tiles is not None:
        t = plan.tiles
        ext.window_tiles(
            *head, segs.tables, segs.cu, t.tile_seg, t.tile_off, t.tile_rows
        )
        if t.rest is None:
            return
        rows, n = t.rest, t.rest.numel()
    nsplit, pa, pm = 0, None, None
    if mfma:
        # fill the chip: splits only from shapes, so captured graphs hold
        groups = n * G * -(-(H // G) * maps // 16)
        most = -(-min(segs.tables.shape[1] * page, window + keep_first + 62) // 128)
        nsplit = max(1, min(-(-512 // groups), 16, most))
        if nsplit > 1:
            cols = n * H * maps * nsplit
            pa, pm = _folded_scratch(q.device, cols * vdim, cols * 2)
    ext.window_rows(*head, segs.row_seg, segs.tables, rows, nsplit, pa, pm)


# -------------------------------------------------- fixed decays, the delta rule
def fixed_decay_kv(q, k, v, decay, H: int, dk: int, dv: int, S, positions, segs,
                   plan: SegmentPlan) -> torch.Tensor:
    """S = decay[h] S + k v^T per head on silu(q), silu(k), silu(v), read out
    by q after the update. q, k, v may be strided and are consumed; S [slots,
    H, dv, dk]."""
    if not q.is_cuda:
        return ref.fixed_decay_kv(q, k, v, decay, H, dk, dv, S, positions, segs)
    y = torch.empty(q.shape[0], H * dv, dtype=q.dtype, device=q.device)
    ext, ch = hybrid_native(), plan.chunks
    args = (y, q, k, v, decay, H, dk, dv, S, positions, segs.cu, segs.slots)
    if ch is not None and dk % 8 == 0 and dv % 8 == 0:
        if ch.short is not None:
            ext.fixed_scan(*args, ch.short)
        for x in (q, k, v):
            ext.silu(x)
        ext.fixed_chunked(*args, *ch.maps)
    else:
        ext.fixed_scan(*args, None)
    return y


def delta_kv(q, k, v, logw, b, H: int, G: int, dk: int, dv: int, S, positions, segs,
             plan: SegmentPlan) -> torch.Tensor:
    """Gated delta rule per head: S = diag(e^logw) S, u = sigmoid(b) (v - S^T
    k), S += k u^T, o = S^T q, on q and k [T, G*dk] divided by their lengths
    (q also by sqrt(dk)); G divides H. q, k, v, b may be strided; logw [T,
    H*dk] fp32 is consumed; S [slots, H, dv, dk]."""
    if not q.is_cuda:
        return ref.delta_kv(q, k, v, logw, b, H, G, dk, dv, S, positions, segs)
    y = torch.empty(q.shape[0], H * dv, dtype=q.dtype, device=q.device)
    ext, ch = hybrid_native(), plan.chunks
    args = (y, q, k, v, logw, b, H, G, dk, dv, S, positions, segs.cu, segs.slots)
    if ch is not None and dk % 8 == 0 and dv % 8 == 0 and dk <= 256:
        if ch.short is not None:
            ext.delta_scan(*args, ch.short)
        ext.delta_chunked(*args, *ch.maps)
    else:
        ext.delta_scan(*args, None)
    return y


from .experts import ExpertSum  # noqa: E402
