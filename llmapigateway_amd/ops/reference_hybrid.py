"""Pure-PyTorch fp32 twins of the hybrid-decoder ops (ops/hybrid.py).

Same role as ops/reference.py: the semantic contract of the HIP kernels and
the CPU engine's compute path. Recurrences are token loops over a segment's
rows; attention gathers its keys from the pages.
"""

from __future__ import annotations

import torch
import torch.nn.functional as F


def build_pair_rope_cache(max_positions, dims, base, device="cpu") -> torch.Tensor:
    """[max_positions, dims] fp32: dims/2 cosines, then dims/2 sines, of
    position * base^(-2i/dims). Angles are taken in float64: at position
    p a fp32 angle is off by up to p * 2^-24."""
    inv = base ** (-torch.arange(0, dims, 2, dtype=torch.float64, device=device) / dims)
    ang = torch.outer(torch.arange(max_positions, dtype=torch.float64, device=device), inv)
    return torch.cat([ang.cos(), ang.sin()], -1).float().contiguous()


def rotate_pairs(x, positions, cos_sin):
    """x [T, ..., dims] fp32, interleaved pairs (2i, 2i+1)."""
    half = cos_sin.shape[1] // 2
    cs = cos_sin[positions].view(-1, *([1] * (x.dim() - 2)), 2 * half)
    c, s = cs[..., :half], cs[..., half:]
    u, v = x[..., 0::2], x[..., 1::2]
    return torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2)


def embed_scaled(tokens, embed, scale, x0):
    x = embed[tokens].float() * scale
    if x0 is not None:
        x0.copy_(x)
    return x


def add_layernorm(x, delta, w, b, eps, dtype, vec, replace):
    if replace:
        x.copy_(delta)
    elif delta is not None:
        x.add_(delta.float())
    if vec is not None:
        x.add_(vec)
    return F.layer_norm(x, (x.shape[-1],), w, b, eps).to(dtype)


def add_cast(x, delta, out):
    if delta is not None:
        x.add_(delta.float())
    out.copy_(x)


def _rms(x, eps):
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def latent_rows(d, q_norm, kv_norm, eps, rot, positions, cos_sin, latent, slot_mapping):
    qr, rank = q_norm.numel(), kv_norm.numel()
    df = d.float()
    cq = _rms(df[:, :qr], eps) * q_norm
    c = _rms(df[:, qr : qr + rank], eps) * kv_norm
    kr = rotate_pairs(df[:, qr + rank :], positions, cos_sin)
    keep = slot_mapping >= 0
    rows = latent.view(-1, latent.shape[-1])
    rows[slot_mapping[keep], : rank + rot] = torch.cat([c, kr], -1)[keep].to(latent.dtype)
    return cq.to(d.dtype)


def fold_queries(q, uk_t, row, positions, cos_sin):
    dim, rank = uk_t.shape[2], uk_t.shape[1]
    T, H, D = q.shape
    out = q.new_zeros(T, H, row)
    out[..., :rank] = torch.einsum("thd,hrd->thr", q[..., :dim].float(), uk_t.float())
    out[..., rank : rank + D - dim] = rotate_pairs(q[..., dim:].float(), positions, cos_sin)
    return out


def latent_attention_folded(ql, latent, rank, sink, scale, positions, segs, row0):
    T, H, row = ql.shape
    out = ql.new_empty(T, H, rank)
    bs = latent.shape[1]
    for t in range(T):
        n = int(positions[t]) + 1
        seg = int(segs.row_seg[row0 + t])
        pages = segs.tables[seg, : (n + bs - 1) // bs].long()
        keys = latent[pages].reshape(-1, row)[:n].float()
        s = ql[t].float() @ keys.T * scale
        p = torch.softmax(torch.cat([s, sink[:, None]], -1), -1)[:, :n]
        out[t] = p @ keys[:, :rank]
    return out


def head_linear(x, w):
    return torch.einsum("thk,hnk->thn", x.float(), w.float()).to(x.dtype).contiguous()


def causal_conv(x, w_t, b, state, positions, segs):
    y = torch.empty(x.shape, dtype=x.dtype)
    k = w_t.shape[0] - 1
    cu = segs.cu.tolist()
    for s, slot in enumerate(segs.slots.tolist()):
        r0, r1 = cu[s], cu[s + 1]
        xs = x[r0:r1].float()
        if slot < 0:
            y[r0:r1] = 0
            continue
        past = state[slot].float()
        if int(positions[r0]) == 0:
            past = torch.zeros_like(past)
        full = torch.cat([past, xs])
        win = full.unfold(0, k + 1, 1)  # [n, C, taps]
        y[r0:r1] = F.silu((win * w_t.t()).sum(-1) + b)
        if k:
            state[slot] = full[-k:].to(state.dtype)
    return y


def ssd(xbc, dt, dt_bias, A_log, D, H, P, N, G, S, positions, segs):
    T = xbc.shape[0]
    xf = xbc.float()
    x = xf[:, : H * P].view(T, H, P)
    Bm = xf[:, H * P : H * P + G * N].view(T, G, N).repeat_interleave(H // G, 1)
    Cm = xf[:, H * P + G * N :].view(T, G, N).repeat_interleave(H // G, 1)
    dt = F.softplus(dt + dt_bias, threshold=1e9)
    decay = torch.exp(-torch.exp(A_log) * dt)
    y = torch.zeros(T, H, P)
    cu = segs.cu.tolist()
    for s, slot in enumerate(segs.slots.tolist()):
        if slot < 0:
            continue
        st = S[slot].clone()  # [H, P, N]
        if int(positions[cu[s]]) == 0:
            st.zero_()
        for t in range(cu[s], cu[s + 1]):
            st = decay[t, :, None, None] * st + (
                (dt[t, :, None] * x[t])[:, :, None] * Bm[t][:, None, :]
            )
            y[t] = (st * Cm[t][:, None, :]).sum(-1) + D[:, None] * x[t]
        S[slot] = st
    return y.view(T, H * P).to(xbc.dtype)


def mlstm(q, k, v, gates, bias, cap, H, dk, dv, S, n, m, positions, segs):
    T = q.shape[0]
    qf = q.float().reshape(T, H, dk) * dk ** -0.5
    kf, vf = k.float().reshape(T, H, dk), v.float().reshape(T, H, dv)
    soft = cap * torch.tanh((gates + bias) / cap)
    i, f = soft[:, :H], F.logsigmoid(soft[:, H:])
    y = torch.zeros(T, H, dv)
    cu = segs.cu.tolist()
    for s, slot in enumerate(segs.slots.tolist()):
        if slot < 0:
            continue
        st, nt, mt = S[slot].clone(), n[slot, 0].clone(), m[slot, 0].clone()
        if int(positions[cu[s]]) == 0:
            st.zero_(), nt.zero_(), mt.zero_()
        for t in range(cu[s], cu[s + 1]):
            m_new = torch.maximum(f[t] + mt, i[t])
            keep, add = torch.exp(f[t] + mt - m_new)[:, None], torch.exp(i[t] - m_new)[:, None]
            mt = m_new
            nt = keep * nt + add * kf[t]
            st = keep[..., None] * st + (add * vf[t])[:, :, None] * kf[t][:, None, :]
            den = torch.maximum((nt * qf[t]).sum(-1).abs(), torch.exp(-mt)) + 1e-6
            y[t] = (st * qf[t][:, None, :]).sum(-1) / den[:, None]
        S[slot], n[slot], m[slot] = st, nt, mt
    return y.view(T, H * dv).to(q.dtype)


def gated_norm(y, gate, w, groups, eps, gate_first):
    T, W = y.shape
    yf, gf = y.float(), gate.float()
    if gate_first:
        yf = yf * F.silu(gf)
    yf = _rms(yf.view(T, groups, W // groups), eps).view(T, W) * w
    if not gate_first:
        yf = yf * torch.sigmoid(gf)
    return yf.to(y.dtype)
