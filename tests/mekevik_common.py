"""Small Mekevik configurations and cases, shared by the CPU and GPU tests."""

from __future__ import annotations

import torch

from lelisun_common import Case, write_checkpoint
from mekevik_oracle import mekevik


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, ff, scale):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top, "scale": scale}}


def attn(heads, kv, dim, vdim, window, far, rows, mlp=None, v_mix=True, mult=3.0):
    # a scale above 1/sqrt(dim) makes single keys stand out
    return {
        "type": "attention", "mlp": mlp, "rows": rows,
        "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
                  "scale": mult * dim ** -0.5, "mask": {"size": window}, "bias_max": far,
                  "v_mix": v_mix},
    }


def config(width, vocab, layers, eps=1e-5, embed=2.0, scale=1.0):
    """``rows`` of a layer stays out of config.json: it is a tensor's size."""
    return {
        "architecture": "Mekevik", "width": width, "vocab": vocab, "layers": layers,
        "embedding": {"scale": embed}, "norm": {"eps": eps}, "logit_scale": scale,
    }


CONFIGS = {
    # sizes that are no multiples of anything: the any-size kernels
    "odd": config(
        70, 211,
        [attn(6, 3, 18, 26, 37, 21, 10, moe(5, 2, 22, 1.5), v_mix=False),
         attn(3, 3, 14, 26, 70, 300, 14, dense(54, 0.6)),
         attn(4, 2, 22, 39, 9, 7, 6),
         attn(2, 1, 10, 78, 1, 5, 4, moe(7, 7, 18, 0.3))],
        eps=1e-3, embed=1.3, scale=0.6,
    ),
    # multiples of 8: the MFMA kernels in most of their sizes; blocks of heads
    # that key heads do not fill; a window beyond the sequence
    "even": config(
        128, 300,
        [attn(8, 2, 40, 64, 50, 40, 16, dense(96, 1.0)),
         attn(16, 4, 72, 32, 33, 90, 24, moe(9, 3, 40, 2.0)),
         attn(24, 8, 16, 16, 64, 33, 8, dense(72, 2.5)),
         attn(32, 8, 136, 16, 31, 64, 32, moe(4, 1, 48, 1.0)),
         attn(40, 2, 24, 64, 1000, 256, 32)],
        eps=1e-5, embed=4.0, scale=1.7,
    ),
    # no layer mixes values; one key head per query head
    "plain": config(
        64, 190,
        [attn(4, 4, 16, 24, 48, 60, 12, dense(64, 1.5), v_mix=False),
         attn(1, 1, 64, 64, 17, 16, 8, moe(4, 2, 64, 3.0), v_mix=False)],
        embed=1.0, scale=1.0,
    ),
    # prompts' tiles of every number of heads a wave
    "tiles": config(
        96, 180,
        [attn(32, 8, 32, 48, 100, 70, 20, dense(64, 1.5)),
         attn(24, 4, 64, 96, 65, 50, 10, moe(6, 2, 32, 1.0)),
         attn(16, 2, 96, 192, 40, 128, 32)],
        eps=1e-6, embed=1.5, scale=2.5,
    ),
}


def tensor_shapes(cfg):
    """Every tensor of a checkpoint and its shape."""
    W, V = cfg["width"], cfg["vocab"]
    s = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
    for i, spec in enumerate(cfg["layers"]):
        m, p = spec["mixer"], f"l{i}.mix."
        H, G = m["heads"], m["kv_heads"]
        s[f"l{i}.norm1"] = (W,)
        s[p + "q"], s[p + "q.norm"] = (H * m["dim"], W), (H * m["dim"],)
        s[p + "k"], s[p + "k.norm"] = (G * m["dim"], W), (G * m["dim"],)
        s[p + "v"], s[p + "g"] = (G * m["vdim"], W), (H * m["vdim"], W)
        s[p + "o"] = (W, H * m["vdim"])
        s[p + "rel"], s[p + "talk"], s[p + "pb"] = (spec["rows"], H), (H, H), (H,)
        if m["v_mix"]:
            s[p + "vmix"] = ()
        if spec["mlp"] is None:
            continue
        e, p = spec["mlp"], f"l{i}.mlp."
        s[f"l{i}.norm2"] = (W,)
        parts = [""]
        if e["kind"] == "moe":
            s[p + "router"] = (e["router"]["experts"], W)
            parts = [f"e{j}." for j in range(e["router"]["experts"])]
        ff = e["ff"] if e["kind"] == "dense" else e["expert"]["ff"]
        for x in parts:
            s[p + x + "gate"] = s[p + x + "up"] = (ff, W)
            s[p + x + "down"] = (W, ff)
    return s


def random_weights(cfg, seed=0):
    """bfloat16 weights whose every mechanism shows in the logits."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        t = torch.randn(shape, generator=g)
        if leaf.startswith("norm"):
            t = 1.0 + 0.2 * t
        elif leaf == "vmix":
            t = 0.4 + 0.2 * t
        elif leaf == "pb":
            t = t - 2.0
        elif leaf == "talk":
            t = torch.eye(shape[0]) + t * shape[0] ** -0.5
        elif leaf == "o":
            t = t * 0.3 * shape[1] ** -0.5
        elif len(shape) == 2 and leaf not in ("rel", "embed"):
            t = t * shape[1] ** -0.5 * (2.0 if name == "head" else 1.0)
        out[name] = t.to(torch.bfloat16)
    return out


class MekevikCase(Case):
    """A configuration with weights on disk, and the oracle's logits."""

    def __init__(self, name, folder, seed=0):
        self.cfg = CONFIGS[name]
        self.weights = random_weights(self.cfg, seed)
        shown = dict(self.cfg, layers=[
            {k: v for k, v in layer.items() if k != "rows"} for layer in self.cfg["layers"]
        ])
        self.path = write_checkpoint(folder, shown, self.weights)
        self._logits = {}

    def expected(self, tokens):
        key = tuple(tokens)
        if key not in self._logits:
            self._logits[key] = mekevik(self.weights, self.cfg, tokens)
        return self._logits[key]
