"""Pure-PyTorch fp32 twins of the hybrid-decoder ops (ops/hybrid.py).

Same role as ops/reference.py: the semantic contract of the HIP kernels and
the CPU engine's compute path. Recurrences are token loops over a segment's
rows; attention gathers its keys from the pages.
"""

from __future__ import annotations

import math

import torch
import torch.nn.functional as F


def build_pair_rope_cache(
    max_positions, dims, base, device="cpu", scaling=None
) -> torch.Tensor:
    """[max_positions, dims] fp32: dims/2 cosines, then dims/2 sines, of
    position * base^(-2i/dims). Angles are taken in float64: at position
    p a fp32 angle is off by up to p * 2^-24.

    scaling (factor, low, high, original): frequencies that turn less than
    ``low`` times within ``original`` positions are divided by ``factor``,
    those that turn more than ``high`` times stay, linear in between."""
    inv = base ** (-torch.arange(0, dims, 2, dtype=torch.float64, device=device) / dims)
    if scaling is not None:
        turns = scaling["original"] * inv / (2.0 * math.pi)
        low, high = scaling["low"], scaling["high"]
        keep = (turns > high).double()
        if high > low:
            keep = ((turns - low) / (high - low)).clamp(0.0, 1.0)
        inv = inv * (keep + (1.0 - keep) / scaling["factor"])
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


# ------------------------------------------------------------- dynamic tanh
def _tanh_norm(x, norm):
    w, b, alpha = norm
    return torch.tanh(alpha * x) * w + b


def add_tanh_norm(x, delta, post, norm, dtype, replace, out):
    if delta is not None:
        d = delta.float()
        if post is not None:
            d = _tanh_norm(d, post)
        x.copy_(d) if replace else x.add_(d)
    y = x if norm is None else _tanh_norm(x, norm)
    if out is None:
        return y.to(dtype)
    out.copy_(y)
    return out


def embed_tanh_norm(tokens, embed, norm, x0):
    x = _tanh_norm(embed[tokens].float(), norm)
    if x0 is not None:
        x0.copy_(x)
    return x


# ---------------------------------------------------- attention over pages
def page_write(k, v, k_pages, v_pages, slot_mapping):
    keep = slot_mapping >= 0
    for rows, pages in ((k, k_pages), (v, v_pages)):
        pages.view(-1, pages.shape[-1])[slot_mapping[keep]] = rows[keep]


def paged_attention(out, q, k_pages, v_pages, H, G, sink, scale, cap, gate, out_scale,
                    positions, segs):
    T, bs = q.shape[0], k_pages.shape[1]
    dim, vdim = k_pages.shape[2] // G, v_pages.shape[2] // G
    for t in range(T):
        n = int(positions[t]) + 1
        pages = segs.tables[int(segs.row_seg[t]), : (n + bs - 1) // bs].long()
        k = k_pages[pages].reshape(-1, G, dim)[:n].float().repeat_interleave(H // G, 1)
        v = v_pages[pages].reshape(-1, G, vdim)[:n].float().repeat_interleave(H // G, 1)
        s = torch.einsum("hd,nhd->hn", q[t].float().view(H, dim), k) * scale
        s = cap * torch.tanh(s / cap)
        p = torch.softmax(torch.cat([s, sink[:, None]], -1), -1)[:, :n]
        o = torch.einsum("hn,nhd->hd", p, v)
        out[t] = (o * (torch.sigmoid(gate[t].float()) * out_scale)[:, None]).view(-1)


# ------------------------------- sigmoid attention over pages, mixed heads
def add_rms_norm(x, deltas, weights, eps, dtype):
    for d in deltas:
        x.add_(d.float())
    unit = _rms(x, eps)
    return tuple((unit * w).to(dtype) for w in weights)


def qkv_rows(q, k, v, q_norm, k_norm, eps, blend, v_first, k_pages, v_pages, slot_mapping):
    vf = v.float()
    if v_first is not None:
        vf = (1.0 - blend) * vf + blend * v_first.float()
    page_write(
        (_rms(k.float(), eps) * k_norm).to(k.dtype), vf.to(v.dtype), k_pages, v_pages,
        slot_mapping,
    )
    return (_rms(q.float(), eps) * q_norm).to(q.dtype)


def sigmoid_attention(out, q, k_pages, v_pages, H, G, scale, bias, talk, window, gate,
                      positions, segs):
    T, bs = q.shape[0], k_pages.shape[1]
    dim, vdim = k_pages.shape[2] // G, v_pages.shape[2] // G
    for t in range(T):
        p = int(positions[t])
        lo = max(0, p - window + 1)
        keys = torch.arange(lo, p + 1)
        slots = segs.tables[int(segs.row_seg[t])].long()[keys // bs] * bs + keys % bs
        k = k_pages.view(-1, G, dim)[slots].float().repeat_interleave(H // G, 1)
        v = v_pages.view(-1, G, vdim)[slots].float().repeat_interleave(H // G, 1)
        s = torch.einsum("hd,nhd->hn", q[t].float().view(H, dim), k) * scale
        s = s + bias[(p - keys).clamp(max=bias.shape[0] - 1), :H].t()
        w = talk.float() @ torch.sigmoid(s)
        o = torch.einsum("hn,nhd->hd", w, v)
        out[t] = o.reshape(-1) * torch.sigmoid(gate[t].float())


# ------------------------------------- recurrences with a decay per channel
def decay_logs(a, w2, bias, kind, tau, rate):
    a = torch.tanh(a.float()) if kind == "exp" else a.float()
    z = a @ w2.float().t() + bias
    if kind == "softplus":
        return -rate * F.softplus(z, threshold=1e9)
    return -torch.exp(z) if kind == "exp" else F.logsigmoid(z) / tau


def token_shift(h, mu, prev, positions, segs):
    hf = h.float()
    last = torch.zeros_like(hf)
    last[1:] = hf[:-1]
    cu = segs.cu.tolist()
    for s, slot in enumerate(segs.slots.tolist()):
        r0 = cu[s]
        fresh = slot < 0 or int(positions[r0]) == 0
        last[r0] = 0.0 if fresh else prev[slot].float()
    for s, slot in enumerate(segs.slots.tolist()):
        if slot >= 0:
            prev[slot] = h[cu[s + 1] - 1]
    return (hf + (last - hf) * mu[:, None]).to(h.dtype)


def decayed_kv(q, k, v, logw, u, qscale, H, dk, dv, S, positions, segs):
    T = q.shape[0]
    qf = q.float().reshape(T, H, dk) * qscale
    kf, vf = k.float().reshape(T, H, dk), v.float().reshape(T, H, dv)
    w = torch.exp(logw).view(T, H, 1, dk)
    y = torch.zeros(T, H, dv)
    cu = segs.cu.tolist()
    for s, slot in enumerate(segs.slots.tolist()):
        if slot < 0:
            continue
        st = S[slot].clone()  # [H, dv, dk]
        if int(positions[cu[s]]) == 0:
            st.zero_()
        for t in range(cu[s], cu[s + 1]):
            if u is not None:
                bonus = (qf[t] * u * kf[t]).sum(-1, keepdim=True)
                y[t] = (st * qf[t][:, None, :]).sum(-1) + bonus * vf[t]
            st = w[t] * st + vf[t][:, :, None] * kf[t][:, None, :]
            if u is None:
                y[t] = (st * qf[t][:, None, :]).sum(-1)
        S[slot] = st
    return y.view(T, H * dv).to(q.dtype)


def head_norm_gate(out, y, gate, w, heads, eps, act):
    T, W = y.shape
    yf = _rms(y.float().view(T, heads, W // heads), eps).view(T, W) * w
    g = gate.float()
    out.copy_(yf * (F.silu(g) if act == "silu" else torch.sigmoid(g)))


# ------------------------------------------------------ hyper-connected streams
def embed_rms_norm(tokens, embed, w, eps):
    return _rms(embed[tokens].float(), eps) * w


def mix_streams(x, pending, coef, rewrite, w, eps, dtype):
    rows = [x[:, s] for s in range(x.shape[1])]
    rows += [y.float() if scale is None else y.float() * scale for y, scale in pending]
    out = torch.einsum("rtw,rc->tcw", torch.stack(rows), coef)
    h = (_rms(out[:, 0], eps) * w).to(dtype)
    return (out[:, 1:].contiguous() if rewrite else x), h


def xielu_(z, pos, neg):
    f = z.float()
    n = f.clamp(max=0)
    return z.copy_(torch.where(f > 0, pos * f * f, neg * (torch.expm1(n) - n)) + 0.5 * f)


# ------------------------- rotary attention in a window, differential or plain
def rotate_halves(x, positions, cos_sin):
    """x [T, heads, D] fp32: dimensions i and i + dims/2 of the first
    dims = cos_sin's width are a pair."""
    half = cos_sin.shape[1] // 2
    cs = cos_sin[positions][:, None]
    c, s = cs[..., :half], cs[..., half:]
    u, v = x[..., :half], x[..., half : 2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half :]], -1)


def rotary_rows(q, k, v, q_norm, k_norm, eps, cos_sin, positions, k_pages, v_pages,
                slot_mapping):
    T, dim = q.shape[0], q_norm.numel()

    def rows(x, w):
        x = _rms(x.float().reshape(T, -1, dim), eps) * w
        return rotate_halves(x, positions, cos_sin).reshape(T, -1).to(q.dtype)

    if k is not None:
        page_write(rows(k, k_norm), v, k_pages, v_pages, slot_mapping)
    return rows(q, q_norm)


def window_attention(out, q, k_pages, v_pages, H, G, maps, scale, window, keep_first, lam, gain,
                     eps, positions, segs):
    T, bs, per = q.shape[0], k_pages.shape[1], H // G
    dim, vdim = k_pages.shape[2] // (G * maps), v_pages.shape[2] // G
    for t in range(T):
        p = int(positions[t])
        lo = max(0, p - window + 1)
        keys = torch.cat([torch.arange(min(lo, keep_first)), torch.arange(lo, p + 1)])
        slots = segs.tables[int(segs.row_seg[t])].long()[keys // bs] * bs + keys % bs
        k = k_pages.view(-1, G, maps, dim)[slots].float().repeat_interleave(per, 1)
        v = v_pages.view(-1, G, vdim)[slots].float().repeat_interleave(per, 1)
        s = torch.einsum("hmd,nhmd->hmn", q[t].float().view(H, maps, dim), k) * scale
        o = torch.einsum("hmn,nhd->hmd", torch.softmax(s, -1), v)
        o = o[:, 0] if maps == 1 else _rms(o[:, 0] - lam * o[:, 1], eps) * gain
        out[t] = o.reshape(-1)


# ----------------------------------------------- fixed decays, the delta rule
def fixed_decay_kv(q, k, v, decay, H, dk, dv, S, positions, segs):
    w = decay.log().clamp(min=-80.0)[:, None].expand(H, dk).reshape(1, -1)
    return decayed_kv(
        F.silu(q.float()), F.silu(k.float()), F.silu(v.float()), w.expand(q.shape[0], -1), None,
        1.0, H, dk, dv, S, positions, segs,
    ).to(q.dtype)


def delta_kv(q, k, v, logw, b, H, G, dk, dv, S, positions, segs):
    T = q.shape[0]

    def unit(x):
        x = x.float().reshape(T, G, dk)
        x = x * torch.rsqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)
        return x.repeat_interleave(H // G, 1)

    qf, kf, vf = unit(q) * dk ** -0.5, unit(k), v.float().reshape(T, H, dv)
    w, beta = torch.exp(logw).view(T, H, 1, dk), torch.sigmoid(b.float())
    y = torch.zeros(T, H, dv)
    cu = segs.cu.tolist()
    for s, slot in enumerate(segs.slots.tolist()):
        if slot < 0:
            continue
        st = S[slot].clone()  # [H, dv, dk]
        if int(positions[cu[s]]) == 0:
            st.zero_()
        for t in range(cu[s], cu[s + 1]):
            st = w[t] * st
            new = beta[t][:, None] * (vf[t] - (st * kf[t][:, None, :]).sum(-1))
            st = st + new[:, :, None] * kf[t][:, None, :]
            y[t] = (st * qf[t][:, None, :]).sum(-1)
        S[slot] = st
    return y.view(T, H * dv).to(q.dtype)


# ------------------------------------------------------------------- experts
def route_experts(z, top):
    e = torch.argsort(z, dim=-1, descending=True, stable=True)[:, :top]
    return e, torch.softmax(z.gather(1, e), -1)


def clamped_glu(x, limit):
    g, u = x.float().chunk(2, -1)
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)).to(x.dtype)


def expert_rows(h, ids, gate_up, down, limit):
    """[T * top, width]: row t * top + j is expert ids[t, j] on row t.
    limit None: silu(gate) * up."""
    T, top = ids.shape
    out = torch.empty(T * top, down.shape[1], dtype=h.dtype)
    flat = ids.reshape(-1)
    for e in flat.unique().tolist():
        rows = torch.nonzero(flat == e).view(-1)
        both = F.linear(h[rows // top], gate_up[e])
        if limit is None:
            g, u = both.float().chunk(2, -1)
            act = (F.silu(g) * u).to(both.dtype)
        else:
            act = clamped_glu(both, limit)
        out[rows] = F.linear(act, down[e])
    return out


def expert_sum(rows, slot, weights, shared):
    y = (rows[slot.long()].float() * weights[..., None]).sum(1)
    return y if shared is None else y + shared.float()


def soft_cap_(x, cap):
    x.div_(cap).tanh_().mul_(cap)
