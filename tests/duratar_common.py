"""Small Duratar configurations and cases, shared by the CPU and GPU tests."""

from __future__ import annotations

import torch

from duratar_oracle import duratar
from lelisun_common import Case, write_checkpoint


def delta(heads, kv, dim, vdim, conv, ra, rg, ff=None):
    """``ra`` and ``rg``, the ranks, stay out of config.json: they are tensors' sizes."""
    return {"type": "channel_delta", "ranks": (ra, rg), "mlp": mlp(ff),
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}}


def attn(heads, kv, dim, vdim, window, keep, rot, base=500.0, scaling=None, diff=0.2,
         kv_from=None, ff=None, mult=2.0):
    # a scale above 1/sqrt(dim) makes single keys stand out
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "diff": diff,
         "scale": mult * dim ** -0.5, "mask": {"size": window, "keep_first": keep},
         "rot": {"base": base, "dims": rot}}
    if scaling is not None:
        m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": mlp(ff)}


def lightning(heads, dim, vdim, decay, ff=None):
    return {"type": "lightning", "mlp": mlp(ff),
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}}


def mlp(ff):
    return {"kind": "dense", "ff": ff} if ff else None


def config(width, vocab, streams, layers, eps=1e-5):
    return {"architecture": "Duratar", "width": width, "vocab": vocab, "streams": streams,
            "layers": layers, "norm": {"eps": eps}}


SCALING = (5.0, 1.0, 6.0, 64)
CONFIGS = {
    # sizes that are no multiples of anything: the any-size kernels; layers
    # without a feed-forward; two layers that read the same layer's keys
    "odd": config(
        70, 211, 3,
        [attn(6, 3, 18, 26, 37, 5, 10, scaling=SCALING, ff=54),
         delta(6, 3, 14, 22, 3, 5, 9),
         attn(6, 3, 18, 26, 11, 0, 10, scaling=SCALING, kv_from=0, diff=0.6),
         lightning(3, 18, 10, (0.9, 0.99, 0.5), ff=50),
         attn(6, 3, 18, 26, 1000, 2, 10, scaling=SCALING, kv_from=0, ff=30, diff=0.05)],
        eps=1e-3,
    ),
    # multiples of 8: the MFMA kernels in several sizes
    "even": config(
        128, 300, 2,
        [delta(4, 2, 40, 64, 4, 16, 24, ff=96), attn(8, 2, 32, 64, 50, 40, 32, ff=72),
         lightning(4, 72, 32, (1.0, 0.999, 0.6, 0.1)), delta(3, 1, 72, 40, 2, 8, 8, ff=64),
         attn(8, 2, 32, 64, 33, 3, 32, kv_from=1, diff=0.7),
         attn(12, 1, 64, 128, 70, 16, 16, scaling=(2.0, 2.0, 3.0, 100), ff=40)],
    ),
    # recurrent layers only, a one-tap convolution, one stream
    "recurrent": config(
        96, 180, 1, [lightning(2, 16, 48, (0.95, 0.7)), delta(2, 2, 128, 96, 1, 8, 16, ff=64),
                     delta(5, 5, 16, 24, 6, 4, 4)],
        eps=1e-2,
    ),
    # attention only: pages are a sequence's whole state
    "attention": config(
        64, 190, 5,
        [attn(4, 4, 16, 24, 48, 1, 8, ff=72), attn(4, 4, 16, 24, 17, 20, 8, kv_from=0),
         attn(2, 1, 128, 136, 60, 4, 128, base=1e4, ff=48)],
        eps=1e-6,
    ),
}


def tensor_shapes(cfg):
    """Every tensor of a checkpoint and its shape."""
    W, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    s = {"embed": (V, W), "head": (V, W), "final.norm": (), "embed.norm": ()}
    for i, spec in enumerate(cfg["layers"]):
        m, p = spec["mixer"], f"l{i}.mix."
        H, dim, vv = m["heads"], m["dim"], m["heads"] * m["vdim"]
        for q in "12"[: 1 + bool(spec["mlp"])]:
            s[f"l{i}.norm{q}"], s[f"l{i}.ls{q}"] = (), (W,)
            s[f"l{i}.hc{q}.in"] = s[f"l{i}.hc{q}.out"] = (S,)
            s[f"l{i}.hc{q}.mix"] = (S, S)
        s[p + "o"] = (W, vv)
        if spec["type"] == "attention":
            G = m["kv_heads"]
            s[p + "q"], s[p + "q.norm"] = (H * 2 * dim, W), (dim,)
            if "kv_from" not in m:
                s[p + "k"], s[p + "k.norm"] = (G * 2 * dim, W), (dim,)
                s[p + "v"] = (G * m["vdim"], W)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                s[p + n] = (dim,)
        elif spec["type"] == "lightning":
            s[p + "q"] = s[p + "k"] = (H * dim, W)
            s[p + "v"] = s[p + "g"] = (vv, W)
            s[p + "norm"] = (vv,)
        else:
            qk, (ra, rg) = m["kv_heads"] * dim, spec["ranks"]
            for n, c in (("q", qk), ("k", qk), ("v", vv)):
                s[p + n], s[f"{p}{n}.conv"] = (c, W), (c, m["conv"])
            s[p + "b"], s[p + "A_log"], s[p + "dt_bias"] = (H, W), (H,), (H * dim,)
            s[p + "a1"], s[p + "a2"] = (ra, W), (H * dim, ra)
            s[p + "g1"], s[p + "g2"], s[p + "norm"] = (rg, W), (vv, rg), (m["vdim"],)
        if spec["mlp"]:
            ff, p = spec["mlp"]["ff"], f"l{i}.mlp."
            s[p + "up"], s[p + "down"], s[p + "act"] = (ff, W), (W, ff), (2,)
    return s


def random_weights(cfg, seed=0):
    """bfloat16 weights whose every mechanism shows in the logits."""
    g = torch.Generator().manual_seed(seed)
    out, S = {}, cfg["streams"]
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        t = torch.randn(shape, generator=g)
        if leaf.startswith(("norm", "ls")):
            t = 1.0 + 0.2 * t
        elif ".hc" in name:
            t = {"in": 1.0 / S + 0.3 * t, "out": 1.0 + 0.4 * t,
                 "mix": torch.eye(S) + 0.25 * t if leaf == "mix" else t}[leaf]
        elif leaf in ("lq1", "lk1", "lq2", "lk2"):
            t = 0.25 * t
        elif leaf == "dt_bias":
            t = t - 2.5
        elif leaf == "A_log":
            t = t - 0.5
        elif leaf == "conv":
            t = t * shape[1] ** -0.5
        elif leaf == "o":
            t = t * 0.5 * shape[1] ** -0.5
        elif leaf == "down":
            t = t * 0.3 * shape[1] ** -0.5
        elif leaf == "b":
            t = 2.0 * t * shape[1] ** -0.5
        elif len(shape) == 2 and leaf != "embed":
            t = t * shape[1] ** -0.5 * (2.0 if name == "head" else 1.0)
        out[name] = t.to(torch.bfloat16)
    return out


class DuratarCase(Case):
    """A configuration with weights on disk, and the oracle's logits."""

    def __init__(self, name, folder, seed=0):
        self.cfg = CONFIGS[name]
        self.weights = random_weights(self.cfg, seed)
        shown = dict(self.cfg, layers=[
            {k: v for k, v in layer.items() if k != "ranks"} for layer in self.cfg["layers"]
        ])
        self.path = write_checkpoint(folder, shown, self.weights)
        self._logits = {}

    def expected(self, tokens):
        key = tuple(tokens)
        if key not in self._logits:
            self._logits[key] = duratar(self.weights, self.cfg, tokens)
        return self._logits[key]
