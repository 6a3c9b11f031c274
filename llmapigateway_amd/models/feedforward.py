"""Feed-forwards of the hybrid decoders, each built from its sizes and
constants and its checkpoint tensors; called with the normed rows, they
return what is to be added to the residual stream: a tensor, or the experts'
parts of it (ops.ExpertSum), which the next stream kernel adds up."""

from __future__ import annotations

from typing import Callable, Dict, Tuple

import torch

from .. import ops
from .twins import add_decode_twins

Getter = Callable[[str], torch.Tensor]


class DenseFF:
    """W_down (silu(W_gate h) * W_up h); with a ``limit`` the clamped GLU of
    the two instead: g = min(W_gate h, limit), u = clamp(W_up h, +-limit),
    g sigmoid(1.702 g) (u + 1)."""

    def __init__(self, m: dict, get: Getter, vec: Getter):
        self.limit = m.get("limit")
        self.w = {"gate_up": torch.cat([get("gate"), get("up")]), "down": get("down")}
        add_decode_twins(self.w, ("gate_up", "down") if self.limit is None else ("down",))

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        ff = m["ff"]
        return {"gate": (ff, width), "up": (ff, width), "down": (width, ff)}

    def __call__(self, h: torch.Tensor) -> torch.Tensor:
        w = self.w
        if self.limit is not None:
            act = ops.clamped_glu(ops.linear(h, w["gate_up"]), float(self.limit))
            return ops.linear(act, w["down"], w.get("down_swz"))
        return ops.linear(
            ops.swiglu_linear(h, w["gate_up"], w.get("gate_up_swz"), w.get("gate_up_int")),
            w["down"], w.get("down_swz"),
        )


class XieluFF:
    """W_down xielu(W_up h): xielu(z) = softplus(p) z^2 + z/2 for z > 0, and
    (1/2 + softplus(q)) (e^z - 1 - z) + z/2 else; p and q are learned."""

    def __init__(self, m: dict, get: Getter, vec: Getter):
        self.w = {"up": get("up"), "down": get("down")}
        p, q = torch.nn.functional.softplus(vec("act").double(), threshold=1e9).tolist()
        self.pos, self.neg = p, 0.5 + q
        add_decode_twins(self.w, ("up", "down"))

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        return {"up": (m["ff"], width), "down": (width, m["ff"]), "act": (2,)}

    def __call__(self, h: torch.Tensor) -> torch.Tensor:
        w = self.w
        z = ops.linear(h, w["up"], w.get("up_swz"))
        return ops.linear(ops.xielu_(z, self.pos, self.neg), w["down"], w.get("down_swz"))


class ExpertFF:
    """Experts of which a router picks ``top`` per token, and optionally a
    shared one for every token. An expert is a DenseFF, with or without a
    limit. Weights: softmax over the chosen logits (which is the softmax over
    all of them, divided by the chosen ones' sum), times the router's
    ``scale``; the router may have a bias."""

    def __init__(self, m: dict, get: Getter, vec: Getter):
        r = m["router"]
        E, self.top, self.scale = r["experts"], r["top"], float(r.get("scale", 1.0))
        self.limit = m["expert"].get("limit")
        self.w_router = get("router")
        self.b_router = vec("router.b") if r.get("bias", True) else None
        self.experts = ops.pack_experts(
            m["expert"]["ff"], self.w_router.shape[1], E,
            lambda e: (get(f"e{e}.gate"), get(f"e{e}.up"), get(f"e{e}.down")),
        )
        self.shared = None
        if m.get("shared") is not None:
            self.shared_limit = float(m["shared"]["limit"])
            self.shared = {
                "gate_up": torch.cat([get("shared.gate"), get("shared.up")]),
                "down": get("shared.down"),
            }
            add_decode_twins(self.shared, ("down",))

    @staticmethod
    def shapes(m: dict, width: int) -> Dict[str, Tuple[int, ...]]:
        E = m["router"]["experts"]
        out: Dict[str, Tuple[int, ...]] = {"router": (E, width)}
        if m["router"].get("bias", True):
            out["router.b"] = (E,)
        parts = [(f"e{e}", m["expert"]["ff"]) for e in range(E)]
        if m.get("shared") is not None:
            parts.append(("shared", m["shared"]["ff"]))
        for name, ff in parts:
            out[f"{name}.gate"] = out[f"{name}.up"] = (ff, width)
            out[f"{name}.down"] = (width, ff)
        return out

    def __call__(self, h: torch.Tensor) -> "ops.ExpertSum":
        routing = ops.route_experts(
            h, self.w_router, self.b_router, self.top, self.experts, self.scale
        )
        rows = ops.expert_rows(h, routing, self.experts, self.limit)
        shared = None
        if self.shared is not None:
            s = self.shared
            act = ops.clamped_glu(ops.linear(h, s["gate_up"]), self.shared_limit)
            shared = ops.linear(act, s["down"], s.get("down_swz"))
        return ops.ExpertSum(rows, routing.slot, routing.weights, shared)


FEEDFORWARDS = {"dense": DenseFF, "xielu": XieluFF, "moe": ExpertFF}
