"""A plain, slow Mekevik: one function per mechanism, whole sequences from
position 0, no batching, no cache.

Everything is float64 on the CPU, written straight from the equations, and
shares no code with llmapigateway_amd. Weights come as a dict of tensors
under their names in the checkpoint; ``cfg`` is the parsed config.json.
"""

from __future__ import annotations

import math

import torch

from filinex_oracle import clamped_expert, sigmoid
from lelisun_oracle import F64, silu, sub, unit_rms


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def bucket(n, rows, far):
    """The table row of a distance n: one each up to half the rows, then
    logarithmically wider ones up to ``far``, beyond which all share the last."""
    half = rows // 2
    if n < half:
        return n
    step = math.log(n / half) / math.log(far / half) * (rows - half)
    return min(rows - 1, half + math.floor(step))


def attention_weights(q, k, scale, rel, far, pb, window):
    """sigmoid weights [H, T, T] of q [T, H, dim] and k [T, G, dim]; 0 where
    the key is not seen."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = torch.zeros(H, T, T, dtype=q.dtype)
    rows = [bucket(n, rel.shape[0], far) for n in range(T)]
    for h in range(H):
        s = q[:, h] @ k[:, h // (H // G)].T * scale
        bias = rel[rows, h]
        for i in range(T):
            lo = max(0, i - window + 1)
            dist = i - torch.arange(lo, i + 1)
            out[h, i, lo : i + 1] = sigmoid(s[i, lo : i + 1] + bias[dist] + pb[h])
    return out


def mix_heads(weights, talk):
    """head h's new weights: sum over g of talk[h, g] weights[g]."""
    H = talk.shape[0]
    return (talk @ weights.reshape(H, -1)).view(weights.shape)


def apply_weights(weights, v):
    """weights [H, T, T] on v [T, G, vdim]: [T, H, vdim]."""
    H, G = weights.shape[0], v.shape[1]
    return torch.stack([weights[h] @ v[:, h // (H // G)] for h in range(H)], 1)


def attention(w, m, eps, h, v_first=None):
    """(output rows, this layer's own values); v_first: the values of the
    first layer that mixes them, None in that layer and in layers that do
    not."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = rms_norm(h @ w["q"].T, w["q.norm"], eps).view(T, H, m["dim"])
    k = rms_norm(h @ w["k"].T, w["k.norm"], eps).view(T, G, m["dim"])
    own = h @ w["v"].T
    v = own
    if v_first is not None:
        v = (1.0 - w["vmix"]) * own + w["vmix"] * v_first
    weights = attention_weights(
        q, k, m["scale"], w["rel"], m["bias_max"], w["pb"], m["mask"]["size"])
    o = apply_weights(mix_heads(weights, w["talk"]), v.view(T, G, m["vdim"]))
    return (o.reshape(T, -1) * sigmoid(h @ w["g"].T)) @ w["o"].T, own


def silu_expert(w, h):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def route(z, top, scale):
    """[(expert, weight), ...] per row of logits z."""
    out = []
    for row in z:
        s = torch.exp(row - row.max())
        s = s / s.sum()
        ids = sorted(range(len(row)), key=lambda e: -float(s[e]))[:top]
        out.append(list(zip(ids, s[ids] / (s[ids].sum() + 1e-20) * scale)))
    return out


def moe(w, m, h):
    r = m["router"]
    y = torch.zeros_like(h)
    for t, chosen in enumerate(route(h @ w["router"].T, r["top"], r["scale"])):
        for e, p in chosen:
            y[t] = y[t] + p * silu_expert(
                {k: w[f"e{e}.{k}"] for k in ("gate", "up", "down")}, h[t])
    return y


def feed_forward(w, m, h):
    return clamped_expert(w, h, m["limit"]) if m["kind"] == "dense" else moe(w, m, h)


def mekevik(weights, cfg, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence; layers_out collects the residual
    stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = weights["embed"].to(F64)[torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    v_first = None
    for i, spec in enumerate(cfg["layers"]):
        w, m = sub(weights, f"l{i}."), spec["mixer"]
        mixes = m["v_mix"]
        y, own = attention(sub(weights, f"l{i}.mix."), m, eps, rms_norm(x, w["norm1"], eps),
                           v_first if mixes else None)
        if mixes and v_first is None:
            v_first = own
        if spec["mlp"] is not None:
            y = y + feed_forward(sub(weights, f"l{i}.mlp."), spec["mlp"],
                                 rms_norm(x, w["norm2"], eps))
        x = x + y
        if layers_out is not None:
            layers_out.append(x.clone())
    x = rms_norm(x, weights["final.norm"].to(F64), eps)
    return x @ weights["head"].to(F64).T * cfg["logit_scale"]
