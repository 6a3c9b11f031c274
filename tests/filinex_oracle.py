"""A plain, slow Filinex: one function per mechanism, one token loop per
recurrence, no batching, no cache, no chunks.

Everything is float64 on the CPU, written straight from the equations, and
shares no code with llmapigateway_amd. Weights come as a dict of tensors
under their names in the checkpoint; ``cfg`` is the parsed config.json.
"""

from __future__ import annotations

import math

import torch

from lelisun_oracle import F64, log_sigmoid, run_order, silu, sub, unit_rms


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def dynamic_tanh(x, w, b, alpha):
    return torch.tanh(alpha * x) * w + b


def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


def softmax_attention(q, k, v, sink, scale, cap):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] of one sequence from
    position 0: capped scores, a sink in the denominator, causal."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        for t in range(T):
            s = soft_cap((k[: t + 1, g] @ q[t, h]) * scale, cap)
            top = torch.maximum(s.max(), sink[h])
            e = torch.exp(s - top)
            out[t, h] = (e @ v[: t + 1, g]) / (e.sum() + torch.exp(sink[h] - top))
    return out


def gated_attention(w, m, eps, h):
    """The left half of 'parallel'."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = (h @ w["q"].T).view(T, H, m["dim"])
    k = (h @ w["k"].T).view(T, G, m["dim"])
    v = (h @ w["v"].T).view(T, G, m["vdim"])
    o = softmax_attention(q, k, v, w["sink"], m["scale"], m["softcap"])
    o = o * sigmoid(h @ w["g"].T)[:, :, None]
    return o.reshape(T, -1) @ w["o"].T


def gla_recurrence(q, k, v, alpha):
    """q, k, alpha [T, H, dk], v [T, H, dv]; q is scaled."""
    T, H, dk = q.shape
    S = torch.zeros(H, dk, v.shape[-1], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        for h in range(H):
            S[h] = alpha[t, h][:, None] * S[h] + torch.outer(k[t, h], v[t, h])
            out[t, h] = S[h].T @ q[t, h]
    return out


def gated_linear_attention(w, m, eps, h):
    """The right half of 'parallel'."""
    T, H, dk, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w["q"].T).view(T, H, dk) * dk ** -0.5
    k = (h @ w["k"].T).view(T, H, dk)
    v = (h @ w["v"].T).view(T, H, dv)
    z = (h @ w["a1"].T) @ w["a2"].T + w["a2.b"]
    alpha = sigmoid(z).view(T, H, dk) ** (1.0 / m["tau"])
    o = unit_rms(gla_recurrence(q, k, v, alpha), eps) * w["norm"]
    return (o.reshape(T, -1) * silu(h @ w["g"].T)) @ w["o"].T


def parallel(w, m, eps, h):
    left = {k[5:]: t for k, t in w.items() if k.startswith("left.")}
    right = {k[6:]: t for k, t in w.items() if k.startswith("right.")}
    return m["left_scale"] * gated_attention(left, m["left"], eps, h) + m[
        "right_scale"
    ] * gated_linear_attention(right, m["right"], eps, h)


def wkv_recurrence(r, k, v, decay, u):
    """r, k, v, decay [T, H, d], u [H, d]."""
    T, H, d = r.shape
    S = torch.zeros(H, d, d, dtype=r.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        for h in range(H):
            kv = torch.outer(k[t, h], v[t, h])
            out[t, h] = (S[h] + u[h][:, None] * kv).T @ r[t, h]
            S[h] = decay[t, h][:, None] * S[h] + kv
    return out


def wkv(w, m, eps, h):
    T, H, d = h.shape[0], m["heads"], m["dim"]
    prev = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    mix = {s: h + (prev - h) * w["mu." + s] for s in "rkvgw"}
    r, k, v = ((mix[s] @ w[s].T).view(T, H, d) for s in "rkv")
    gate = silu(mix["g"] @ w["g"].T)
    decay = torch.exp(-torch.exp(torch.tanh(mix["w"] @ w["w1"].T) @ w["w2"].T + w["w0"]))
    o = wkv_recurrence(r, k, v, decay.view(T, H, d), w["u"])
    return (unit_rms(o, eps).reshape(T, H * d) * w["norm"] * gate) @ w["o"].T


def clamped_expert(w, h, limit):
    g = torch.clamp(h @ w["gate"].T, max=limit)
    u = torch.clamp(h @ w["up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w["down"].T


def route(z, top):
    """[(expert, weight), ...] per row of logits z."""
    out = []
    for row in z:
        ids = sorted(range(len(row)), key=lambda e: -float(row[e]))[:top]
        e = torch.exp(row[ids] - row[ids].max())
        out.append(list(zip(ids, e / e.sum())))
    return out


def moe(w, m, h):
    y = torch.zeros_like(h)
    for t, chosen in enumerate(route(h @ w["router"].T + w["router.b"], m["router"]["top"])):
        for e, p in chosen:
            part = {k: w[f"e{e}.{k}"] for k in ("gate", "up", "down")}
            y[t] = y[t] + p * clamped_expert(part, h[t], m["expert"]["limit"])
    shared = {k: w[f"shared.{k}"] for k in ("gate", "up", "down")}
    return y + clamped_expert(shared, h, m["shared"]["limit"])


MIXERS = {"parallel": parallel, "wkv": wkv}


def norm(w, name, x):
    return dynamic_tanh(x, w[name], w[name + ".b"], w[name + ".alpha"])


def filinex(weights, cfg, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence; layers_out collects the residual
    stream after every layer run."""
    eps = cfg["norm"]["eps"]
    W = {k: weights[k].to(F64) for k in (
        "embed", "embed.norm", "embed.norm.b", "embed.norm.alpha", "head",
        "final.norm", "final.norm.b", "final.norm.alpha")}
    x = norm(W, "embed.norm", W["embed"][torch.as_tensor(tokens)])
    x0 = x
    for i, t in run_order(cfg):
        spec, p = cfg["layers"][i], f"l{i}."
        w = sub(weights, p)
        if t is not None:
            x = torch.cat([x, x0], -1) @ weights["loop.in"].to(F64).T
        mixer = MIXERS[spec["type"]](sub(weights, p + "mix."), spec["mixer"], eps,
                                     norm(w, "norm1", x))
        x = x + norm(w, "norm1b", mixer)
        if spec["mlp"] is not None:
            x = x + norm(w, "norm2b", moe(sub(weights, p + "mlp."), spec["mlp"],
                                          norm(w, "norm2", x)))
        if layers_out is not None:
            layers_out.append(x.clone())
    return soft_cap(norm(W, "final.norm", x) @ W["head"].T, cfg["logit_softcap"])
