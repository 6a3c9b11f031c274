"""A plain, slow Lelisun: one function per mechanism, one token loop per
recurrence, no batching, no cache, no chunks.

Everything is float64 on the CPU, written straight from the equations, and
shares no code with llmapigateway_amd: the tests compare the framework's
layers, schedules and kernels with it. Weights come as a dict of tensors
under their names in the checkpoint; ``cfg`` is the parsed config.json.
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def log_sigmoid(z):
    return -softplus(-z)


def rotate_pairs(x, pos, base, dims):
    """x [T, ..., D]; dims 2i and 2i+1 turn by pos * base^(-2i/dims)."""
    out = x.clone()
    for i in range(dims // 2):
        a = pos.to(F64) * base ** (-2.0 * i / dims)
        a = a.reshape([-1] + [1] * (x.dim() - 2))
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., 2 * i + 1] = v * torch.cos(a) + u * torch.sin(a)
    return out


def latent_attention(w, m, eps, h):
    """Causal attention with a sink over keys and values unfolded from the
    latent; h [T, width] are all tokens of one sequence from position 0."""
    T, H = h.shape[0], m["heads"]
    dim, rd, vd, rank = m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(T)
    base, rdims = m["rot"]["base"], m["rot"]["dims"]
    c_q = unit_rms(h @ w["dq"].T, eps) * w["dq.norm"]
    q = (c_q @ w["uq"].T).view(T, H, dim + rd)
    qn, qr = q[..., :dim], rotate_pairs(q[..., dim:], pos, base, rdims)
    dkv = h @ w["dkv"].T
    c = unit_rms(dkv[:, :rank], eps) * w["dkv.norm"]
    kr = rotate_pairs(dkv[:, rank:], pos, base, rdims)
    kn = (c @ w["uk"].T).view(T, H, dim)
    v = (c @ w["uv"].T).view(T, H, vd)
    out = torch.zeros(T, H, vd, dtype=h.dtype)
    for hd in range(H):
        s = (qn[:, hd] @ kn[:, hd].T + qr[:, hd] @ kr.T) * m["scale"]
        s = s.masked_fill(torch.ones(T, T).triu(1).bool(), -math.inf)
        top = torch.maximum(s.max(-1).values, w["sink"][hd])
        e = torch.exp(s - top[:, None])
        out[:, hd] = (e @ v[:, hd]) / (
            e.sum(-1) + torch.exp(w["sink"][hd] - top)
        )[:, None]
    return out.reshape(T, H * vd) @ w["o"].T


def mlstm_recurrence(q, k, v, i, f):
    """q, k [T, H, dim] (q scaled), v [T, H, vdim], log gates [T, H]."""
    T, H, dk = q.shape
    S = torch.zeros(H, dk, v.shape[-1], dtype=q.dtype)
    n = torch.zeros(H, dk, dtype=q.dtype)
    m = torch.zeros(H, dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        m_new = torch.maximum(f[t] + m, i[t])
        keep, add = torch.exp(f[t] + m - m_new), torch.exp(i[t] - m_new)
        S = keep[:, None, None] * S + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + add[:, None] * k[t]
        m = m_new
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = (S * q[t][:, :, None]).sum(1) / den[:, None]
    return out


def mlstm(w, m, eps, h):
    T, H, dk, dv, cap = h.shape[0], m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q = (h @ w["q"].T).view(T, H, dk) / math.sqrt(dk)
    k = (h @ w["k"].T).view(T, H, dk)
    v = (h @ w["v"].T).view(T, H, dv)
    i = cap * torch.tanh((h @ w["i"].T + w["i.b"]) / cap)
    f = log_sigmoid(cap * torch.tanh((h @ w["f"].T + w["f.b"]) / cap))
    o = unit_rms(mlstm_recurrence(q, k, v, i, f), eps).reshape(T, H * dv)
    return (o * w["norm"] * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def causal_conv(x, w, b):
    """x [T, C], w [C, taps] with the current token's tap last."""
    T, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x) + b
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                y[t] = y[t] + w[:, j] * x[s]
    return y


def mamba2_recurrence(x, B, C, dt, A_log, D):
    """x [T, H, P], B, C [T, G, N], dt [T, H] (after softplus)."""
    T, H, P = x.shape
    G, N = B.shape[1:]
    S = torch.zeros(H, N, P, dtype=x.dtype)
    y = torch.zeros_like(x)
    for t in range(T):
        for hd in range(H):
            g = hd // (H // G)
            S[hd] = torch.exp(-torch.exp(A_log[hd]) * dt[t, hd]) * S[hd] + dt[
                t, hd
            ] * torch.outer(B[t, g], x[t, hd])
            y[t, hd] = C[t, g] @ S[hd] + D[hd] * x[t, hd]
    return y


def mamba2(w, m, eps, h):
    T, H, P, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, xbc, dt = (h @ w["in"].T).split([inner, inner + 2 * G * N, H], -1)
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x, B, C = xbc.split([inner, G * N, G * N], -1)
    y = mamba2_recurrence(
        x.view(T, H, P), B.view(T, G, N), C.view(T, G, N),
        softplus(dt + w["dt_bias"]), w["A_log"], w["D"],
    )
    y = (y.reshape(T, inner) * silu(z)).view(T, m["norm_groups"], -1)
    return (unit_rms(y, eps).reshape(T, inner) * w["norm"]) @ w["o"].T


def dense_ff(w, h):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


MIXERS = {"latent_attention": latent_attention, "mlstm": mlstm, "mamba2": mamba2}


def sub(weights, prefix):
    return {k[len(prefix):]: t.to(F64) for k, t in weights.items() if k.startswith(prefix)}


def run_order(cfg):
    """[(layer, pass or None)]: pass t at the first layer of loop pass t."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    order = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        order += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
    return order + [(i, None) for i in range(lp["stop"], n)]


def lelisun(weights, cfg, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence; layers_out collects the residual
    stream after every layer run."""
    eps = cfg["norm"]["eps"]
    W = {k: t.to(F64) for k, t in weights.items() if not k.startswith("l") or k.startswith("loop")}
    x = W["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    x0 = x
    for i, t in run_order(cfg):
        spec, p = cfg["layers"][i], f"l{i}."
        w = sub(weights, p)
        if t is not None:
            x = torch.cat([x, x0], -1) @ W["loop.in"].T + W["loop.step"][t]
        h = layer_norm(x, w["norm1"], w["norm1.b"], eps)
        x = x + MIXERS[spec["type"]](sub(weights, p + "mix."), spec["mixer"], eps, h)
        if spec["mlp"] is not None:
            h = layer_norm(x, w["norm2"], w["norm2.b"], eps)
            x = x + dense_ff(sub(weights, p + "mlp."), h)
        if layers_out is not None:
            layers_out.append(x.clone())
    x = layer_norm(x, W["final.norm"], W["final.norm.b"], eps)
    return x @ W["head"].T


def tensor_shapes(cfg):
    """Every tensor of a checkpoint and its shape."""
    width, vocab = cfg["width"], cfg["vocab"]
    s = {"embed": (vocab, width), "final.norm": (width,), "final.norm.b": (width,),
         "head": (vocab, width)}
    if cfg.get("loop"):
        s["loop.in"] = (width, 2 * width)
        s["loop.step"] = (cfg["loop"]["times"], width)
    for i, spec in enumerate(cfg["layers"]):
        m, p = spec["mixer"], f"l{i}.mix."
        s[f"l{i}.norm1"] = s[f"l{i}.norm1.b"] = (width,)
        H = m["heads"]
        if spec["type"] == "latent_attention":
            s[p + "dq"], s[p + "dq.norm"] = (m["q_rank"], width), (m["q_rank"],)
            s[p + "uq"] = (H * (m["dim"] + m["rot_dim"]), m["q_rank"])
            s[p + "dkv"] = (m["kv_rank"] + m["rot_dim"], width)
            s[p + "dkv.norm"] = (m["kv_rank"],)
            s[p + "uk"], s[p + "uv"] = (H * m["dim"], m["kv_rank"]), (H * m["vdim"], m["kv_rank"])
            s[p + "sink"], s[p + "o"] = (H,), (width, H * m["vdim"])
        elif spec["type"] == "mamba2":
            inner, gn = H * m["vdim"], m["groups"] * m["state"]
            s[p + "in"] = (2 * inner + 2 * gn + H, width)
            s[p + "conv"], s[p + "conv.b"] = (inner + 2 * gn, m["conv"]), (inner + 2 * gn,)
            s[p + "dt_bias"] = s[p + "A_log"] = s[p + "D"] = (H,)
            s[p + "norm"], s[p + "o"] = (inner,), (width, inner)
        else:
            s[p + "q"] = s[p + "k"] = (H * m["dim"], width)
            s[p + "v"] = s[p + "g"] = (H * m["vdim"], width)
            s[p + "i"] = s[p + "f"] = (H, width)
            s[p + "i.b"] = s[p + "f.b"] = (H,)
            s[p + "norm"], s[p + "o"] = (H * m["vdim"],), (width, H * m["vdim"])
        if spec["mlp"] is not None:
            ff = spec["mlp"]["ff"]
            s[f"l{i}.norm2"] = s[f"l{i}.norm2.b"] = (width,)
            s[f"l{i}.mlp.gate"] = s[f"l{i}.mlp.up"] = (ff, width)
            s[f"l{i}.mlp.down"] = (width, ff)
    return s


def random_weights(cfg, seed=0):
    """bfloat16 weights whose every mechanism shows in the logits."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".", 1)[-1]
        t = torch.randn(shape, generator=g)
        if len(shape) == 2:
            t = t * shape[1] ** -0.5 * (1.5 if leaf.endswith((".uq", ".dq")) else 1.0)
        if name == "embed":
            t = t / cfg["embedding"]["scale"] * cfg["width"] ** 0.5
        if leaf.endswith("norm") or leaf in ("norm1", "norm2") or leaf.endswith(".D"):
            t = 1.0 + 0.2 * t
        elif leaf.endswith("conv"):
            t = t * shape[1] ** 0.5
        elif leaf.endswith("dt_bias"):
            t = t - 1.0
        elif leaf.endswith("A_log"):
            t = 0.7 * t
        elif leaf.endswith("f.b"):
            t = t + 3.0
        elif leaf.endswith(("norm.b", "norm1.b", "norm2.b", "conv.b")):
            t = 0.2 * t
        out[name] = t.to(torch.bfloat16)
    return out
