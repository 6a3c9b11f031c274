"""Token mixers of the hybrid decoders, each built from its sizes and
constants and its checkpoint tensors.

A mixer reads the normed rows of a flat batch, keeps what it must remember
in its own cache view (pages for attention, one state slot per sequence for
recurrences; engine/kvcache.py allocates them from ``cache_spec``) and
returns the rows to be added to the residual stream. Projections that read
the same rows are stacked into one product. What enters a recurrence (gate
and step-size pre-activations) leaves its product in fp32.
"""

from __future__ import annotations

from typing import Callable, Dict, NamedTuple, Tuple

import torch

from .. import ops
from .batch import ForwardBatch
from .twins import add_decode_twins

Getter = Callable[[str], torch.Tensor]


class CacheSpec(NamedTuple):
    """What one run of a layer keeps: ``pages`` name -> row width (one row
    per token, compute dtype); ``state`` name -> (shape, fp32?) per
    sequence slot."""

    pages: Dict[str, int]
    state: Dict[str, Tuple[Tuple[int, ...], bool]]


def _pad8(n: int) -> int:
    return (n + 7) // 8 * 8


def _stack(parts):
    """Weights [n, width] stacked to one, every part at a multiple of 8 rows
    and all of it a multiple of 64 (zero rows in between); the parts' row
    ranges by name."""
    rows, cut, at = [], {}, 0
    for i, (name, w) in enumerate(parts):
        cut[name] = (at, at + w.shape[0])
        end = (at + w.shape[0] + 7) // 8 * 8
        if i + 1 == len(parts):
            end = (end + 63) // 64 * 64
        rows += [w, w.new_zeros(end - cut[name][1], w.shape[1])]
        at = end
    return torch.cat(rows), cut


class LatentAttention:
    """Attention whose keys and values unfold from one cached latent per
    token, plus one rotated key part that all heads share; the softmax has
    a learned sink per head in its denominator.

    Two equivalent forms: folded (queries are taken into the latent space,
    scores and sums run over the cached rows themselves; decode and short
    portions) and unfolded (per-head keys and values are made from the
    latents; long portions)."""

    plans = ("unfold",)  # what it uses of a step's plan

    def __init__(self, m: dict, eps: float, get: Getter, vec: Getter, rope: Callable):
        self.m, self.eps = m, eps
        self.H, self.dim, self.rot = m["heads"], m["dim"], m["rot_dim"]
        self.vdim, self.rank, self.q_rank = m["vdim"], m["kv_rank"], m["q_rank"]
        self.scale = float(m["scale"])
        self.row = _pad8(self.rank + self.rot)  # cached row, zero-padded
        self.cos_sin = rope(m["rot"]["base"], m["rot"]["dims"])
        self.q_norm, self.kv_norm = vec("dq.norm"), vec("dkv.norm")
        self.sink = vec("sink")
        uk = get("uk").view(self.H, self.dim, self.rank)
        uv = get("uv")
        self.w = {
            "down": torch.cat([get("dq"), get("dkv")]),
            "uq": get("uq"),
            "ukv": torch.cat([uk.reshape(-1, self.rank), uv]),
            "o": get("o"),
        }
        self.uk_t = uk.transpose(1, 2).contiguous()            # [H, rank, dim]
        self.uv = uv.view(self.H, self.vdim, self.rank)        # [H, vdim, rank]
        self.unfolds = ops.can_unfold(self.dim, self.rot, self.vdim, self.rank)
        add_decode_twins(self.w, ("down", "uq", "o"))

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        H = m["heads"]
        return {
            "dq": (m["q_rank"], width), "dq.norm": (m["q_rank"],),
            "uq": (H * (m["dim"] + m["rot_dim"]), m["q_rank"]),
            "dkv": (m["kv_rank"] + m["rot_dim"], width), "dkv.norm": (m["kv_rank"],),
            "uk": (H * m["dim"], m["kv_rank"]), "uv": (H * m["vdim"], m["kv_rank"]),
            "sink": (H,), "o": (width, H * m["vdim"]),
        }

    @staticmethod
    def cache_spec(m: dict, width: int) -> CacheSpec:
        return CacheSpec({"latent": _pad8(m["kv_rank"] + m["rot_dim"])}, {})

    def __call__(self, h: torch.Tensor, batch: ForwardBatch, cache, plan) -> torch.Tensor:
        T, w = h.shape[0], self.w
        d = ops.linear(h, w["down"], w.get("down_swz"))
        latent = cache["latent"]
        cq = ops.latent_rows(
            d, self.q_norm, self.kv_norm, self.eps, self.rot,
            batch.positions, self.cos_sin, latent, batch.slot_mapping,
        )
        q = ops.linear(cq, w["uq"], w.get("uq_swz")).view(T, self.H, self.dim + self.rot)
        if plan.unfold is not None and self.unfolds:
            out = ops.latent_attention_unfolded(
                q, latent, w["ukv"], self.sink, self.scale, self.dim, self.vdim,
                self.rank, self.cos_sin, batch.positions, plan.unfold,
            )
            Tu = plan.unfold.rows
            if Tu < T:
                out[Tu:] = self._folded(q[Tu:], latent, batch, Tu)
        else:
            out = self._folded(q, latent, batch, 0)
        return ops.linear(out.view(T, self.H * self.vdim), w["o"], w.get("o_swz"))

    def _folded(self, q, latent, batch, row0: int) -> torch.Tensor:
        pos = batch.positions[row0:]
        ql = ops.fold_queries(q, self.uk_t, self.row, self.cos_sin, pos)
        o = ops.latent_attention_folded(
            ql, latent, self.rank, self.sink, self.scale, pos, batch.segs,
            row0,
        )
        return ops.head_linear(o, self.uv)


class Mamba2:
    """State-space duality layer: short causal convolution, scalar decay
    per head, B and C shared by the heads of a group, gated group norm."""

    plans = ("chunks",)  # what it uses of a step's plan

    def __init__(self, m: dict, eps: float, get: Getter, vec: Getter, rope: Callable):
        self.m, self.eps = m, eps
        self.H, self.P, self.N, self.G = m["heads"], m["vdim"], m["state"], m["groups"]
        self.inner = self.H * self.P
        self.norm_groups = m["norm_groups"]
        w_in = get("in")
        self.w = {"in": w_in[: -self.H].contiguous(), "o": get("o")}
        self.w_dt = w_in[-self.H :].contiguous()
        self.conv_t = vec("conv").t().contiguous()  # [taps, channels]
        self.conv_b = vec("conv.b")
        self.dt_bias, self.A_log, self.D = vec("dt_bias"), vec("A_log"), vec("D")
        self.norm = vec("norm")
        add_decode_twins(self.w, ("in", "o"))

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        H, inner, gn = m["heads"], m["heads"] * m["vdim"], m["groups"] * m["state"]
        return {
            "in": (2 * inner + 2 * gn + H, width), "conv": (inner + 2 * gn, m["conv"]),
            "conv.b": (inner + 2 * gn,), "dt_bias": (H,), "A_log": (H,), "D": (H,),
            "norm": (inner,), "o": (width, inner),
        }

    @staticmethod
    def cache_spec(m: dict, width: int) -> CacheSpec:
        channels = m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]
        return CacheSpec({}, {
            "S": ((m["heads"], m["vdim"], m["state"]), True),
            "conv": ((m["conv"] - 1, channels), False),
        })

    def __call__(self, h: torch.Tensor, batch: ForwardBatch, cache, plan) -> torch.Tensor:
        w = self.w
        u = ops.linear(h, w["in"], w.get("in_swz"))
        dt = ops.linear_f32(h, self.w_dt)
        xbc = ops.causal_conv(
            u[:, self.inner :], self.conv_t, self.conv_b, cache["conv"],
            batch.positions, batch.segs, plan,
        )
        y = ops.ssd(
            xbc, dt, self.dt_bias, self.A_log, self.D, self.H, self.P, self.N, self.G,
            cache["S"], batch.positions, batch.segs, plan,
        )
        y = ops.gated_norm(
            y, u[:, : self.inner], self.norm, self.norm_groups, self.eps, gate_first=True
        )
        return ops.linear(y, w["o"], w.get("o_swz"))


class MLSTM:
    """Matrix-memory recurrence with exponential gates kept in range by a
    running maximum, a normaliser state, head-wise norm and output gate."""

    plans = ("chunks",)  # what it uses of a step's plan

    def __init__(self, m: dict, eps: float, get: Getter, vec: Getter, rope: Callable):
        self.m, self.eps = m, eps
        self.H, self.dk, self.dv = m["heads"], m["dim"], m["vdim"]
        self.cap = float(m["gate_cap"])
        self.w = {
            "qkvg": torch.cat([get("q"), get("k"), get("v"), get("g")]),
            "o": get("o"),
        }
        self.w_if = torch.cat([get("i"), get("f")])
        self.if_bias = torch.cat([vec("i.b"), vec("f.b")])
        self.norm = vec("norm")
        add_decode_twins(self.w, ("qkvg", "o"))

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        H, dk, dv = m["heads"], m["dim"], m["vdim"]
        return {
            "q": (H * dk, width), "k": (H * dk, width), "v": (H * dv, width),
            "g": (H * dv, width), "o": (width, H * dv), "norm": (H * dv,),
            "i": (H, width), "i.b": (H,), "f": (H, width), "f.b": (H,),
        }

    @staticmethod
    def cache_spec(m: dict, width: int) -> CacheSpec:
        H, dk, dv = m["heads"], m["dim"], m["vdim"]
        return CacheSpec({}, {
            # every tile of 64 value rows carries its own n and m
            "S": ((H, dv, dk), True), "n": ((-(-dv // 64), H, dk), True),
            "m": ((-(-dv // 64), H), True),
        })

    def __call__(self, h: torch.Tensor, batch: ForwardBatch, cache, plan) -> torch.Tensor:
        w, kq, vv = self.w, self.H * self.dk, self.H * self.dv
        u = ops.linear(h, w["qkvg"], w.get("qkvg_swz"))
        gates = ops.linear_f32(h, self.w_if)
        y = ops.mlstm(
            u[:, :kq], u[:, kq : 2 * kq], u[:, 2 * kq : 2 * kq + vv], gates,
            self.if_bias, self.cap, self.H, self.dk, self.dv,
            cache["S"], cache["n"], cache["m"], batch.positions, batch.segs, plan,
        )
        y = ops.gated_norm(
            y, u[:, 2 * kq + vv :], self.norm, self.H, self.eps, gate_first=False
        )
        return ops.linear(y, w["o"], w.get("o_swz"))


class GatedAttention:
    """Grouped-query attention without rotation: soft-capped scores, a
    learned sink per head in the softmax's denominator, and a sigmoid gate
    per head on its output. Leaves the heads' outputs in the rows it is
    given; the projections around it belong to the mixer that holds it."""

    def __init__(self, m: dict, get: Getter, vec: Getter, out_scale: float):
        self.H, self.G, self.dim, self.vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        self.scale, self.cap = float(m["scale"]), float(m["softcap"])
        self.sink, self.out_scale = vec("sink"), out_scale

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        H, G = m["heads"], m["kv_heads"]
        return {
            "q": (H * m["dim"], width), "k": (G * m["dim"], width),
            "v": (G * m["vdim"], width), "sink": (H,), "g": (H, width),
            "o": (width, H * m["vdim"]),
        }

    @staticmethod
    def cache_spec(m: dict, width: int) -> CacheSpec:
        return CacheSpec({"k": m["kv_heads"] * m["dim"], "v": m["kv_heads"] * m["vdim"]}, {})

    def __call__(self, q, k, v, gate, out, batch: ForwardBatch, cache, plan) -> None:
        ops.page_write(k, v, cache["k"], cache["v"], batch.slot_mapping)
        ops.paged_attention(
            out, q, cache["k"], cache["v"], self.H, self.G, self.sink, self.scale, self.cap,
            gate, self.out_scale, batch.positions, batch.segs, plan,
        )


class SigmoidAttention:
    """Grouped-query attention over the last ``window`` tokens without
    rotation or softmax: a key weighs sigmoid(score + a learned bias of its
    distance and the head), and learned mixes of all heads' weights go to the
    values. Queries and keys are normed over all heads at once; every output
    value has a sigmoid gate. Layers with ``v_mix``, after the first of them,
    blend their values with the first one's."""

    plans = ("head_tiles",)  # what it uses of a step's plan

    def __init__(self, m: dict, eps: float, get: Getter, vec: Getter, rope: Callable):
        self.H, self.G, self.eps = m["heads"], m["kv_heads"], eps
        self.scale, self.window, self.v_mix = float(m["scale"]), m["window"], m.get("v_mix")
        w_in, self.cut = _stack([(n, get(n)) for n in ("q", "k", "v", "g")])
        self.w = {"in": w_in, "o": get("o")}
        self.q_norm, self.k_norm = vec("q.norm"), vec("k.norm")
        self.talk = get("talk")
        self.bias = ops.distance_bias(vec("rel"), vec("pb"), m["bias_max"], self.window)
        self.blend = float(vec("vmix")) if self.v_mix else 0.0
        add_decode_twins(self.w, ("in", "o"))

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        H, G = m["heads"], m["kv_heads"]
        out: Dict[str, Tuple[int, ...]] = {
            "q": (H * m["dim"], width), "k": (G * m["dim"], width),
            "v": (G * m["vdim"], width), "q.norm": (H * m["dim"],),
            "k.norm": (G * m["dim"],), "rel": (m["bias_rows"], H), "talk": (H, H), "pb": (H,),
            "g": (H * m["vdim"], width), "o": (width, H * m["vdim"]),
        }
        if m.get("v_mix"):
            out["vmix"] = ()
        return out

    @staticmethod
    def cache_spec(m: dict, width: int) -> CacheSpec:
        return CacheSpec({"k": m["kv_heads"] * m["dim"], "v": m["kv_heads"] * m["vdim"]}, {})

    def __call__(self, h: torch.Tensor, batch: ForwardBatch, cache, plan) -> torch.Tensor:
        w = self.w
        u = ops.linear(h, w["in"], w.get("in_swz"))
        q, k, v, g = (u[:, lo:hi] for lo, hi in self.cut.values())
        first = None
        if self.v_mix:
            first = plan.carry.get("v_first")
            if first is None:
                plan.carry["v_first"] = v
        q = ops.qkv_rows(
            q, k, v, self.q_norm, self.k_norm, self.eps, self.blend, first, cache["k"],
            cache["v"], batch.slot_mapping,
        )
        out = torch.empty(h.shape[0], w["o"].shape[1], dtype=h.dtype, device=h.device)
        ops.sigmoid_attention(
            out, q, cache["k"], cache["v"], self.H, self.G, self.scale, self.bias, self.talk,
            self.window, g, batch.positions, batch.segs, plan,
        )
        return ops.linear(out, w["o"], w.get("o_swz"))


class GatedLinearAttention:
    """Linear attention with a decay per key channel, sigmoid(z)^(1/tau) of a
    low-rank projection z, head-wise RMS norm and a silu gate."""

    def __init__(self, m: dict, eps: float, get: Getter, vec: Getter, out_scale: float):
        self.H, self.dk, self.dv, self.eps = m["heads"], m["dim"], m["vdim"], eps
        self.tau = float(m["tau"])
        self.a2, self.a2_bias = get("a2"), vec("a2.b")
        # the norm's weight, shared by the heads, takes the output's scale
        self.norm = (vec("norm") * out_scale).repeat(self.H)

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        kk, vv, rank = m["heads"] * m["dim"], m["heads"] * m["vdim"], m["decay_rank"]
        return {
            "q": (kk, width), "k": (kk, width), "v": (vv, width), "g": (vv, width),
            "o": (width, vv), "norm": (m["vdim"],), "a1": (rank, width), "a2": (kk, rank),
            "a2.b": (kk,),
        }

    @staticmethod
    def cache_spec(m: dict, width: int) -> CacheSpec:
        return CacheSpec({}, {"S": ((m["heads"], m["vdim"], m["dim"]), True)})

    def __call__(self, q, k, v, gate, a, out, batch: ForwardBatch, cache, plan) -> None:
        logw = ops.decay_logs(a, self.a2, self.a2_bias, "sigmoid", self.tau)
        y = ops.decayed_kv(
            q, k, v, logw, None, self.dk ** -0.5, self.H, self.dk, self.dv, cache["S"],
            batch.positions, batch.segs, plan,
        )
        ops.head_norm_gate(out, y, gate, self.norm, self.H, self.eps)


class Parallel:
    """Gated attention (left) and gated linear attention (right) side by
    side on the same rows: one product projects for both, and one product of
    their joined outputs, each scaled already, sums both output projections."""

    plans = ("tiles", "chunks")  # what it uses of a step's plan

    def __init__(self, m: dict, eps: float, get: Getter, vec: Getter, rope: Callable):
        def side(f, name):
            return lambda n: f(f"{name}.{n}")

        gl, gr = side(get, "left"), side(get, "right")
        self.left = GatedAttention(m["left"], gl, side(vec, "left"), float(m["left_scale"]))
        self.right = GatedLinearAttention(
            m["right"], eps, gr, side(vec, "right"), float(m["right_scale"])
        )
        w_in, self.cut = _stack([
            ("q", gl("q")), ("k", gl("k")), ("v", gl("v")), ("rq", gr("q")), ("rk", gr("k")),
            ("rv", gr("v")), ("rg", gr("g")), ("a", gr("a1")), ("g", gl("g")),
        ])
        o_l, o_r = gl("o"), gr("o")
        self.n_left, self.n_right = o_l.shape[1], o_r.shape[1]
        pad = _pad8(self.n_left) - self.n_left  # the right half starts aligned
        self.w = {
            "in": w_in, "o": torch.cat([o_l, o_l.new_zeros(o_l.shape[0], pad), o_r], 1),
        }
        add_decode_twins(self.w, ("in", "o"))

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        out = {f"left.{k}": s for k, s in GatedAttention.shapes(m["left"], width).items()}
        for k, s in GatedLinearAttention.shapes(m["right"], width).items():
            out[f"right.{k}"] = s
        return out

    @staticmethod
    def cache_spec(m: dict, width: int) -> CacheSpec:
        left = GatedAttention.cache_spec(m["left"], width)
        right = GatedLinearAttention.cache_spec(m["right"], width)
        return CacheSpec({**left.pages, **right.pages}, {**left.state, **right.state})

    def __call__(self, h: torch.Tensor, batch: ForwardBatch, cache, plan) -> torch.Tensor:
        w = self.w
        u = ops.linear(h, w["in"], w.get("in_swz"))
        p = {name: u[:, lo:hi] for name, (lo, hi) in self.cut.items()}
        K = w["o"].shape[1]
        both = torch.empty(h.shape[0], K, dtype=h.dtype, device=h.device)
        if K != self.n_left + self.n_right:
            both.zero_()  # the columns between the halves
        self.left(p["q"], p["k"], p["v"], p["g"], both[:, : self.n_left], batch, cache, plan)
        self.right(
            p["rq"], p["rk"], p["rv"], p["rg"], p["a"], both[:, K - self.n_right :],
            batch, cache, plan,
        )
        return ops.linear(both, w["o"], w.get("o_swz"))


class WKV:
    """RWKV-style time mixing: five projections of different blends of a
    token's row and the one before it; a data-dependent decay per key channel,
    exp(-exp(.)), and an extra weight u on the current token's own key."""

    plans = ("chunks",)  # what it uses of a step's plan

    def __init__(self, m: dict, eps: float, get: Getter, vec: Getter, rope: Callable):
        self.H, self.d, self.eps = m["heads"], m["dim"], eps
        self.mu = torch.stack([vec(f"mu.{s}") for s in "rkvgw"])
        self.w = {s: get(s) for s in ("r", "k", "v", "g", "w1", "o")}
        self.w2, self.w0, self.u = get("w2"), vec("w0"), vec("u")
        self.norm = vec("norm")
        add_decode_twins(self.w, ("r", "k", "v", "g", "o"))

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        n, rank = m["heads"] * m["dim"], m["decay_rank"]
        out: Dict[str, Tuple[int, ...]] = {f"mu.{s}": (width,) for s in "rkvgw"}
        out.update({s: (n, width) for s in "rkvg"})
        out.update({
            "w1": (rank, width), "w2": (n, rank), "w0": (n,), "u": (m["heads"], m["dim"]),
            "norm": (n,), "o": (width, n),
        })
        return out

    @staticmethod
    def cache_spec(m: dict, width: int) -> CacheSpec:
        return CacheSpec({}, {
            "S": ((m["heads"], m["dim"], m["dim"]), True), "prev": ((width,), False),
        })

    def __call__(self, h: torch.Tensor, batch: ForwardBatch, cache, plan) -> torch.Tensor:
        w = self.w
        mixes = ops.token_shift(h, self.mu, cache["prev"], batch.positions, batch.segs)
        r, k, v, g = (ops.linear(mixes[i], w[s], w.get(s + "_swz")) for i, s in enumerate("rkvg"))
        logw = ops.decay_logs(ops.linear(mixes[4], w["w1"]), self.w2, self.w0, "exp", 1.0)
        y = ops.decayed_kv(
            r, k, v, logw, self.u, 1.0, self.H, self.d, self.d, cache["S"],
            batch.positions, batch.segs, plan,
        )
        out = torch.empty_like(y)
        ops.head_norm_gate(out, y, g, self.norm, self.H, self.eps)
        return ops.linear(out, w["o"], w.get("o_swz"))


class RotaryAttention:
    """Grouped-query softmax attention over the last ``window`` tokens and the
    first ``keep_first`` ones; queries and keys are RMS-normed per head and
    rotated in halves on their first ``rot.dims`` dimensions. With ``diff`` it
    is differential: every head has two maps of queries and keys over the same
    values, and gives unit_rms(map 1 - lambda map 2) (1 - diff). With
    ``kv_from`` its keys and values are another layer's, out of that layer's
    cache."""

    plans = ("tiles",)  # what it uses of a step's plan

    def __init__(self, m: dict, eps: float, get: Getter, vec: Getter, rope: Callable):
        self.H, self.G, self.dim, self.eps = m["heads"], m["kv_heads"], m["dim"], eps
        self.scale, self.window, self.keep = float(m["scale"]), m["window"], m["keep_first"]
        self.own = m.get("kv_from") is None
        w_in, self.cut = _stack([(n, get(n)) for n in ("qkv" if self.own else "q")])
        self.w = {"in": w_in, "o": get("o")}
        self.q_norm, self.k_norm = vec("q.norm"), vec("k.norm") if self.own else None
        self.cos_sin = rope(m["rot"]["base"], m["rot"]["dims"], m["rot"].get("scaling"))
        self.maps, self.lam, self.gain = 1, 0.0, 1.0
        if m.get("diff") is not None:
            l1, l2 = (float((vec("lq" + n).double() * vec("lk" + n).double()).sum().exp())
                      for n in "12")
            self.maps, self.lam = 2, l1 - l2 + m["diff"]
            self.gain = 1.0 - m["diff"]
        add_decode_twins(self.w, ("in", "o"))

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        maps = 2 if m.get("diff") is not None else 1
        H, G, dim = m["heads"], m["kv_heads"], m["dim"]
        out: Dict[str, Tuple[int, ...]] = {
            "q": (H * maps * dim, width), "q.norm": (dim,), "o": (width, H * m["vdim"]),
        }
        if m.get("kv_from") is None:
            out.update({
                "k": (G * maps * dim, width), "v": (G * m["vdim"], width), "k.norm": (dim,),
            })
        if maps == 2:
            out.update({n: (dim,) for n in ("lq1", "lk1", "lq2", "lk2")})
        return out

    @staticmethod
    def cache_spec(m: dict, width: int) -> CacheSpec:
        if m.get("kv_from") is not None:
            return CacheSpec({}, {})
        maps, G = 2 if m.get("diff") is not None else 1, m["kv_heads"]
        return CacheSpec({"k": G * maps * m["dim"], "v": G * m["vdim"]}, {})

    def __call__(self, h: torch.Tensor, batch: ForwardBatch, cache, plan) -> torch.Tensor:
        w = self.w
        u = ops.linear(h, w["in"], w.get("in_swz"))
        p = {name: u[:, lo:hi] for name, (lo, hi) in self.cut.items()}
        q = ops.rotary_rows(
            p["q"], p.get("k"), p.get("v"), self.q_norm, self.k_norm, self.eps, self.cos_sin,
            batch.positions, cache["k"], cache["v"], batch.slot_mapping,
        )
        out = torch.empty(h.shape[0], w["o"].shape[1], dtype=h.dtype, device=h.device)
        ops.window_attention(
            out, q, cache["k"], cache["v"], self.H, self.G, self.maps, self.scale, self.window,
            self.keep, self.lam, self.gain, self.eps, batch.positions, batch.segs, plan,
        )
        return ops.linear(out, w["o"], w.get("o_swz"))


class Lightning:
    """Linear attention with a fixed decay per head on silu'd queries, keys
    and values; one RMS norm over all heads' outputs and a sigmoid gate."""

    plans = ("chunks",)  # what it uses of a step's plan

    def __init__(self, m: dict, eps: float, get: Getter, vec: Getter, rope: Callable):
        self.H, self.dk, self.dv, self.eps = m["heads"], m["dim"], m["vdim"], eps
        w_in, self.cut = _stack([(n, get(n)) for n in "qkvg"])
        self.w = {"in": w_in, "o": get("o")}
        self.norm = vec("norm")
        self.decay = torch.tensor(m["decay"], dtype=torch.float32, device=self.norm.device)
        add_decode_twins(self.w, ("in", "o"))

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        kk, vv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
        return {
            "q": (kk, width), "k": (kk, width), "v": (vv, width), "g": (vv, width),
            "o": (width, vv), "norm": (vv,),
        }

    @staticmethod
    def cache_spec(m: dict, width: int) -> CacheSpec:
        return CacheSpec({}, {"S": ((m["heads"], m["vdim"], m["dim"]), True)})

    def __call__(self, h: torch.Tensor, batch: ForwardBatch, cache, plan) -> torch.Tensor:
        w = self.w
        u = ops.linear(h, w["in"], w.get("in_swz"))
        q, k, v, g = (u[:, lo:hi] for lo, hi in self.cut.values())
        y = ops.fixed_decay_kv(
            q, k, v, self.decay, self.H, self.dk, self.dv, cache["S"], batch.positions,
            batch.segs, plan,
        )
        y = ops.gated_norm(y, g, self.norm, 1, self.eps, gate_first=False)
        return ops.linear(y, w["o"], w.get("o_swz"))


class ChannelDelta:
    """Gated delta rule with a decay per key channel: short convolutions on
    queries, keys and values, unit queries and keys, decays and output gates
    from low-rank projections, a head-wise RMS norm."""

    plans = ("chunks",)  # what it uses of a step's plan

    def __init__(self, m: dict, eps: float, get: Getter, vec: Getter, rope: Callable):
        self.H, self.G, self.eps = m["heads"], m["kv_heads"], eps
        self.dk, self.dv = m["dim"], m["vdim"]
        w_in, self.cut = _stack([(n, get(n)) for n in ("q", "k", "v", "a1", "g1", "b")])
        self.w = {"in": w_in, "g2": get("g2"), "o": get("o")}
        # the convolutions of q, k and v are one over their stacked columns
        taps = w_in.new_zeros(self.cut["v"][1], m["conv"], dtype=torch.float32)
        for n in "qkv":
            taps[self.cut[n][0] : self.cut[n][1]] = vec(n + ".conv")
        self.conv_t = taps.t().contiguous()
        self.conv_b = torch.zeros_like(self.conv_t[0])
        self.a2, self.dt_bias = get("a2"), vec("dt_bias")
        self.rate = vec("A_log").exp().repeat_interleave(self.dk)
        self.norm = vec("norm").repeat(self.H)  # shared by the heads
        add_decode_twins(self.w, ("in", "o"))

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        H, qk, vv = m["heads"], m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
        ra, rg, taps = m["decay_rank"], m["gate_rank"], m["conv"]
        return {
            "q": (qk, width), "k": (qk, width), "v": (vv, width), "q.conv": (qk, taps),
            "k.conv": (qk, taps), "v.conv": (vv, taps), "b": (H, width), "A_log": (H,),
            "a1": (ra, width), "a2": (H * m["dim"], ra), "dt_bias": (H * m["dim"],),
            "g1": (rg, width), "g2": (vv, rg), "norm": (m["vdim"],), "o": (width, vv),
        }

    @staticmethod
    def cache_spec(m: dict, width: int) -> CacheSpec:
        channels = 2 * _pad8(m["kv_heads"] * m["dim"]) + m["heads"] * m["vdim"]
        return CacheSpec({}, {
            "S": ((m["heads"], m["vdim"], m["dim"]), True),
            "conv": ((m["conv"] - 1, channels), False),
        })

    def __call__(self, h: torch.Tensor, batch: ForwardBatch, cache, plan) -> torch.Tensor:
        w, cut = self.w, self.cut
        u = ops.linear(h, w["in"], w.get("in_swz"))
        x = ops.causal_conv(
            u[:, : cut["v"][1]], self.conv_t, self.conv_b, cache["conv"], batch.positions,
            batch.segs, plan,
        )
        a, g1, b = (u[:, slice(*cut[n])] for n in ("a1", "g1", "b"))
        logw = ops.decay_logs(a, self.a2, self.dt_bias, "softplus", rate=self.rate)
        q, k, v = (x[:, slice(*cut[n])] for n in "qkv")
        y = ops.delta_kv(
            q, k, v, logw, b, self.H, self.G, self.dk, self.dv, cache["S"], batch.positions,
            batch.segs, plan,
        )
        gate = ops.linear(g1, w["g2"])
        out = torch.empty_like(y)
        ops.head_norm_gate(out, y, gate, self.norm, self.H, self.eps, act="sigmoid")
        return ops.linear(out, w["o"], w.get("o_swz"))


MIXERS = {
    "latent_attention": LatentAttention, "mamba2": Mamba2, "mlstm": MLSTM,
    "parallel": Parallel, "wkv": WKV, "sigmoid_attention": SigmoidAttention,
    "rotary_attention": RotaryAttention, "lightning": Lightning, "channel_delta": ChannelDelta,
}
