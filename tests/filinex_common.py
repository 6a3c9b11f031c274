"""Small Filinex configurations and cases, shared by the CPU and GPU tests."""

from __future__ import annotations

import torch

from filinex_oracle import filinex
from lelisun_common import Case, write_checkpoint


def moe(experts, top, ff, limit, shared_ff, shared_limit):
    return {
        "kind": "moe", "router": {"experts": experts, "top": top},
        "expert": {"ff": ff, "limit": limit}, "shared": {"ff": shared_ff, "limit": shared_limit},
    }


def par(heads, kv, dim, vdim, cap, lin_heads, lin_dim, lin_vdim, tau, scales, rank, mlp=None,
        mult=3.0):
    # a scale above 1/sqrt(dim) makes single keys stand out in the softmax
    return {
        "type": "parallel", "mlp": mlp, "rank": rank,
        "mixer": {
            "left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
                     "scale": mult * dim ** -0.5, "softcap": cap},
            "right": {"heads": lin_heads, "dim": lin_dim, "vdim": lin_vdim, "tau": tau},
            "left_scale": scales[0], "right_scale": scales[1],
        },
    }


def wkv(heads, dim, rank, mlp=None):
    return {"type": "wkv", "mlp": mlp, "rank": rank, "mixer": {"heads": heads, "dim": dim}}


def config(width, vocab, layers, loop=None, eps=1e-5, cap=20.0):
    """``rank`` of a layer stays out of config.json: it is a tensor's size."""
    return {
        "architecture": "Filinex", "width": width, "vocab": vocab, "layers": layers,
        "norm": {"eps": eps}, "logit_softcap": cap,
        "loop": dict(zip(("start", "stop", "times"), loop)) if loop else None,
    }


CONFIGS = {
    # sizes that are no multiples of anything: the any-size kernels
    "odd": config(
        70, 211,
        [wkv(3, 14, 5, moe(5, 2, 22, 1.5, 30, 0.7)),
         par(6, 3, 18, 26, 2.5, 3, 10, 22, 8.0, (0.7, 1.3), 7, mult=8.0),
         wkv(2, 22, 9, moe(7, 1, 18, 2.5, 26, 3.0))],
        loop=(1, 3, 2), eps=1e-3, cap=9.0,
    ),
    # multiples of 8: the MFMA kernels, several tiles and slices of each; a
    # group of more than 16 heads; a cap that needs the running maximum
    "even": config(
        128, 300,
        [par(20, 5, 40, 72, 8.0, 2, 136, 200, 16.0, (1.2, 0.8), 16, moe(9, 3, 40, 1.0, 56, 2.0)),
         wkv(2, 72, 24, moe(9, 9, 72, 2.0, 24, 0.5)),
         par(18, 1, 136, 16, 50.0, 5, 24, 40, 2.0, (0.5, 1.5), 8)],
        loop=(0, 2, 3), eps=1e-5, cap=30.0,
    ),
    # recurrent layers only, one expert, no loop
    "recurrent": config(
        96, 180, [wkv(4, 24, 8, moe(1, 1, 48, 7.0, 32, 7.0)), wkv(1, 64, 16)], eps=1e-4, cap=15.0,
    ),
    # one key head per query head, one of each; looped once, from the first layer on
    "plain": config(
        64, 190,
        [par(4, 4, 16, 24, 30.0, 1, 32, 64, 1.0, (1.0, 1.0), 4, moe(4, 2, 64, 1.0, 64, 1.0)),
         par(1, 1, 64, 64, 12.0, 4, 16, 16, 32.0, (2.0, 0.25), 12)],
        loop=(0, 1, 1), cap=50.0,
    ),
}


def tensor_shapes(cfg):
    """Every tensor of a checkpoint and its shape."""
    width, vocab = cfg["width"], cfg["vocab"]
    s = {"embed": (vocab, width), "head": (vocab, width)}

    def norm(name):
        s[name] = s[name + ".b"] = (width,)
        s[name + ".alpha"] = ()

    norm("embed.norm"), norm("final.norm")
    if cfg.get("loop"):
        s["loop.in"] = (width, 2 * width)
    for i, spec in enumerate(cfg["layers"]):
        m, p, rank = spec["mixer"], f"l{i}.mix.", spec["rank"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if spec["mlp"] else ()):
            norm(f"l{i}.{n}")
        if spec["type"] == "parallel":
            a, b, q = m["left"], m["right"], p + "left."
            s[q + "q"] = (a["heads"] * a["dim"], width)
            s[q + "k"] = (a["kv_heads"] * a["dim"], width)
            s[q + "v"] = (a["kv_heads"] * a["vdim"], width)
            s[q + "sink"], s[q + "g"] = (a["heads"],), (a["heads"], width)
            s[q + "o"] = (width, a["heads"] * a["vdim"])
            kk, vv, q = b["heads"] * b["dim"], b["heads"] * b["vdim"], p + "right."
            s[q + "q"] = s[q + "k"] = (kk, width)
            s[q + "v"] = s[q + "g"] = (vv, width)
            s[q + "o"], s[q + "norm"] = (width, vv), (b["vdim"],)
            s[q + "a1"], s[q + "a2"], s[q + "a2.b"] = (rank, width), (kk, rank), (kk,)
        else:
            n = m["heads"] * m["dim"]
            for x in "rkvgw":
                s[p + "mu." + x] = (width,)
            for x in "rkvg":
                s[p + x] = (n, width)
            s[p + "w1"], s[p + "w2"], s[p + "w0"] = (rank, width), (n, rank), (n,)
            s[p + "u"], s[p + "norm"], s[p + "o"] = (m["heads"], m["dim"]), (n,), (width, n)
        if spec["mlp"]:
            e, p = spec["mlp"], f"l{i}.mlp."
            E = e["router"]["experts"]
            s[p + "router"], s[p + "router.b"] = (E, width), (E,)
            for x, ff in [(f"e{j}", e["expert"]["ff"]) for j in range(E)] + [
                ("shared", e["shared"]["ff"])
            ]:
                s[f"{p}{x}.gate"] = s[f"{p}{x}.up"] = (ff, width)
                s[f"{p}{x}.down"] = (width, ff)
    return s


def random_weights(cfg, seed=0):
    """bfloat16 weights whose every mechanism shows in the logits."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        t = torch.randn(shape, generator=g)
        if ".mu." in name:
            t = 0.5 + 0.4 * t
        elif leaf == "alpha":
            t = 0.8 + 0.2 * t
        elif leaf == "w0":
            t = t - 1.5
        elif leaf.startswith("norm"):
            t = 1.0 + 0.2 * t
        elif name.endswith("a2.b"):
            t = t + 2.0
        elif leaf == "b":
            t = 0.3 * t
        elif name == "embed":
            pass
        elif len(shape) == 2 and leaf != "u":
            t = t * shape[1] ** -0.5 * (2.0 if name == "head" else 1.0)
        out[name] = t.to(torch.bfloat16)
    return out


class FilinexCase(Case):
    """A configuration with weights on disk, and the oracle's logits."""

    def __init__(self, name, folder, seed=0):
        self.cfg = CONFIGS[name]
        self.weights = random_weights(self.cfg, seed)
        shown = dict(self.cfg, layers=[
            {k: v for k, v in layer.items() if k != "rank"} for layer in self.cfg["layers"]
        ])
        self.path = write_checkpoint(folder, shown, self.weights)
        self._logits = {}

    def expected(self, tokens):
        key = tuple(tokens)
        if key not in self._logits:
            self._logits[key] = filinex(self.weights, self.cfg, tokens)
        return self._logits[key]
