"""A plain, slow Duratar: one function per mechanism, one token loop per
recurrence, whole sequences from position 0, no batching, no cache.

Everything is float64 on the CPU, written straight from the equations, and
shares no code with llmapigateway_amd. Weights come as a dict of tensors
under their names in the checkpoint; ``cfg`` is the parsed config.json.
"""

from __future__ import annotations

import math

import torch

from filinex_oracle import sigmoid
from lelisun_oracle import F64, silu, softplus, sub, unit_rms


# ------------------------------------------------------------------ the stream
def read_streams(streams, w_in):
    """sum_s w_in[s] streams[s]: streams [S, T, W]."""
    return sum(w_in[s] * streams[s] for s in range(len(streams)))


def write_streams(streams, mix, w_out, y):
    """stream t <- sum_s mix[s, t] stream s + w_out[t] y, all from the old ones."""
    S = len(streams)
    return torch.stack([
        sum(mix[s, t] * streams[s] for s in range(S)) + w_out[t] * y for t in range(S)
    ])


def xielu(z, p, q):
    """softplus(p) z^2 + z/2 above 0, (1/2 + softplus(q)) (e^z - 1 - z) + z/2 below."""
    neg = torch.clamp(z, max=0)
    low = (0.5 + softplus(q)) * (torch.exp(neg) - 1.0 - neg) + 0.5 * z
    return torch.where(z > 0, softplus(p) * z * z + 0.5 * z, low)


def feed_forward(w, h):
    return xielu(h @ w["up"].T, w["act"][0], w["act"][1]) @ w["down"].T


# ------------------------------------------------------------------- attention
def frequencies(rot):
    """The angle per position of every pair of dimensions."""
    out = []
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        c = rot.get("scaling")
        if c is not None:
            ratio = c["original"] * f / (2.0 * math.pi)  # original / wavelength
            if ratio < c["low"]:
                f = f / c["factor"]
            elif ratio <= c["high"]:
                s = (ratio - c["low"]) / (c["high"] - c["low"])
                f = (1.0 - s) * f / c["factor"] + s * f
        out.append(f)
    return out


def rotate_half(x, rot):
    """x [T, ..., D]: dimensions i and i + dims/2 turn by position * frequency."""
    out, half = x.clone(), rot["dims"] // 2
    pos = torch.arange(x.shape[0], dtype=F64).reshape([-1] + [1] * (x.dim() - 2))
    for i, f in enumerate(frequencies(rot)):
        c, s = torch.cos(pos * f), torch.sin(pos * f)
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def visible(T, window, keep_first):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    return (j <= i) & ((i - j < window) | (j < keep_first))


def softmax_map(q, k, v, scale, seen):
    """One map of one head: q [T, dim], k [T, dim], v [T, vdim]."""
    s = (q @ k.T * scale).masked_fill(~seen, -math.inf)
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return (e / e.sum(-1, keepdim=True)) @ v


def lambda_of(w, diff):
    return (torch.exp((w["lq1"] * w["lk1"]).sum()) - torch.exp((w["lq2"] * w["lk2"]).sum())
            + diff)


def combine_maps(a1, a2, lam, diff, eps):
    return unit_rms(a1 - lam * a2, eps) * (1.0 - diff)


def keys_and_values(w, m, eps, h):
    """k [T, G, 2, dim] normed and rotated, v [T, G, vdim]."""
    T, G = h.shape[0], m["kv_heads"]
    k = unit_rms((h @ w["k"].T).view(T, G, 2, m["dim"]), eps) * w["k.norm"]
    return rotate_half(k, m["rot"]), (h @ w["v"].T).view(T, G, m["vdim"])


def attention(w, m, eps, h, kv=None):
    """(output rows, the keys and values used); kv: another layer's."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    if kv is None:
        kv = keys_and_values(w, m, eps, h)
    k, v = kv
    q = unit_rms((h @ w["q"].T).view(T, H, 2, m["dim"]), eps) * w["q.norm"]
    q = rotate_half(q, m["rot"])
    seen = visible(T, m["mask"]["size"], m["mask"]["keep_first"])
    lam, out = lambda_of(w, m["diff"]), []
    for hd in range(H):
        g = hd // (H // G)
        a1, a2 = (softmax_map(q[:, hd, i], k[:, g, i], v[:, g], m["scale"], seen) for i in (0, 1))
        out.append(combine_maps(a1, a2, lam, m["diff"], eps))
    return torch.cat(out, -1) @ w["o"].T, kv


# ----------------------------------------------------------------- recurrences
def lightning_recurrence(q, k, v, decay):
    """q, k [T, H, dim], v [T, H, vdim]: S <- decay S + k v^T, o = S^T q."""
    T, H, dim = q.shape
    S = torch.zeros(H, dim, v.shape[2], dtype=q.dtype)
    out = torch.zeros_like(v)
    d = torch.as_tensor(decay, dtype=q.dtype)[:, None, None]
    for t in range(T):
        S = d * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def lightning(w, m, eps, h):
    T, H = h.shape[0], m["heads"]
    q, k = (silu(h @ w[n].T).view(T, H, m["dim"]) for n in "qk")
    v = silu(h @ w["v"].T).view(T, H, m["vdim"])
    o = lightning_recurrence(q, k, v, m["decay"]).reshape(T, -1)
    return (unit_rms(o, eps) * w["norm"] * sigmoid(h @ w["g"].T)) @ w["o"].T


def causal_conv(x, taps):
    """silu of sum_j taps[c, j] x[t - (n - 1) + j, c], zeros before the start."""
    n = taps.shape[1]
    full = torch.cat([torch.zeros(n - 1, x.shape[1], dtype=x.dtype), x])
    return silu(sum(full[j : j + x.shape[0]] * taps[:, j] for j in range(n)))


def unit_vectors(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def channel_decay(a, w2, dt_bias, A_log, H):
    """exp(-exp(A_log) softplus(w2 a + dt_bias)): [T, H, dim]."""
    z = softplus(a @ w2.T + dt_bias).view(a.shape[0], H, -1)
    return torch.exp(-torch.exp(A_log)[:, None] * z)


def delta_recurrence(q, k, v, g, beta):
    """q, k, g [T, H, dim], v [T, H, vdim], beta [T, H]: S <- g S,
    u = beta (v - S^T k), S <- S + k u^T, o = S^T q."""
    T, H, dim = q.shape
    S = torch.zeros(H, dim, v.shape[2], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def channel_delta(w, m, eps, h):
    T, H, K, dim = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k, v = (causal_conv(h @ w[n].T, w[n + ".conv"]) for n in "qkv")
    q, k = (unit_vectors(x.view(T, K, dim)).repeat_interleave(H // K, 1) for x in (q, k))
    g = channel_decay(h @ w["a1"].T, w["a2"], w["dt_bias"], w["A_log"], H)
    o = delta_recurrence(q * dim ** -0.5, k, v.view(T, H, -1), g, sigmoid(h @ w["b"].T))
    gate = sigmoid((h @ w["g1"].T) @ w["g2"].T)
    return ((unit_rms(o, eps) * w["norm"]).reshape(T, -1) * gate) @ w["o"].T


# ------------------------------------------------------------------- the model
def duratar(weights, cfg, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence; layers_out collects the sum of the
    streams after every layer."""
    eps = cfg["norm"]["eps"]
    weights = {k: t.to(F64) for k, t in weights.items()}
    x = unit_rms(weights["embed"][torch.as_tensor(tokens)], eps) * weights["embed.norm"]
    streams, kvs = torch.stack([x] * cfg["streams"]), {}
    for i, spec in enumerate(cfg["layers"]):
        w, m = sub(weights, f"l{i}."), spec["mixer"]
        mw = sub(weights, f"l{i}.mix.")
        h = unit_rms(read_streams(streams, w["hc1.in"]), eps) * w["norm1"]
        if spec["type"] == "attention":
            y, kvs[i] = attention(mw, m, eps, h, kvs.get(m.get("kv_from")))
        else:
            y = {"lightning": lightning, "channel_delta": channel_delta}[spec["type"]](
                mw, m, eps, h)
        streams = write_streams(streams, w["hc1.mix"], w["hc1.out"], y * w["ls1"])
        if spec["mlp"] is not None:
            h = unit_rms(read_streams(streams, w["hc2.in"]), eps) * w["norm2"]
            y = feed_forward(sub(weights, f"l{i}.mlp."), h)
            streams = write_streams(streams, w["hc2.mix"], w["hc2.out"], y * w["ls2"])
        if layers_out is not None:
            layers_out.append(streams.sum(0))
    x = unit_rms(streams.sum(0), eps) * weights["final.norm"]
    return x @ weights["head"].T
