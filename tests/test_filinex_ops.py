"""Each mechanism of Filinex alone, against the float64 oracle: the CPU ops in
fp32, the gfx950 kernels in fp32 and bf16."""

import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).resolve().parent))

import filinex_oracle as oracle  # noqa: E402
from test_lelisun_ops import BF16, F32, Pool, close, every, rand  # noqa: E402
from llmapigateway_amd import ops  # noqa: E402
from llmapigateway_amd.ops import experts as X  # noqa: E402


def f64(t):
    return t.double().cpu()


# ------------------------------------------------------------------ the stream
@every
@pytest.mark.parametrize("width", [7, 96, 1000, 4096])
def test_stream_add_and_dynamic_tanh(device, dtype, width):
    x = rand(5, width, seed=1, device=device, mult=2.0)
    d = rand(5, width, seed=2, device=device, dtype=dtype)
    full = rand(5, width, seed=3, device=device)
    post = (rand(width, seed=5, device=device), rand(width, seed=6, device=device), 0.7)
    norm = (rand(width, seed=7, device=device), rand(width, seed=8, device=device), -1.3)
    dt = lambda t, n: oracle.dynamic_tanh(f64(t), f64(n[0]), f64(n[1]), n[2])  # noqa: E731

    y = x.clone()
    close(ops.add_tanh_norm(y, None, None, norm, dtype), dt(x, norm), dtype)
    assert torch.equal(y, x)
    stream = f64(x) + dt(d, post)
    close(ops.add_tanh_norm(y, d, post, norm, dtype), dt(stream, norm), dtype)
    close(y, stream, F32, 5)
    close(ops.add_tanh_norm(y, full, None, norm, dtype, replace=True), dt(full, norm), dtype)
    assert torch.equal(y, full)
    both = torch.zeros(5, 2 * width, dtype=dtype, device=device)
    ops.add_tanh_norm(y, d, post, None, dtype, out=both[:, :width])
    close(y, f64(full) + dt(d, post), F32, 5)
    assert torch.equal(both[:, :width], y.to(dtype)) and not both[:, width:].any()


@every
def test_small_arguments_keep_their_precision(device, dtype):
    """tanh of arguments around 1e-4 .. 0.3, relative to themselves."""
    x = torch.logspace(-4, -0.5, 64, device=device).view(8, 8).contiguous()
    one, zero = torch.ones(8, device=device), torch.zeros(8, device=device)
    y = ops.add_tanh_norm(x, None, None, (one, zero, 1.0), dtype)
    assert ((f64(y) / torch.tanh(f64(x)) - 1).abs() < (5e-3 if dtype == BF16 else 2e-6)).all()


@every
@pytest.mark.parametrize("width", [7, 128])
def test_embedding_norm(device, dtype, width):
    e = rand(50, width, seed=1, device=device, dtype=dtype)
    norm = (rand(width, seed=7, device=device), rand(width, seed=8, device=device), 1.7)
    tok = torch.tensor([3, 49, 0, 3], device=device)
    both = torch.zeros(4, 2 * width, dtype=dtype, device=device)
    x = ops.embed_tanh_norm(tok, e, norm, both[:, width:])
    close(x, oracle.dynamic_tanh(f64(e[tok]), f64(norm[0]), f64(norm[1]), 1.7), F32, 5)
    assert torch.equal(both[:, width:], x.to(dtype)) and not both[:, :width].any()


@every
@pytest.mark.parametrize("n", [1, 5, 1023, 70000])
def test_logit_cap(device, dtype, n):
    x = rand(n, seed=n, device=device, mult=20.0)
    want = oracle.soft_cap(f64(x), 11.0)
    ops.soft_cap_(x, 11.0)
    close(x[None], want[None], F32)


@every
@pytest.mark.parametrize("heads,gs", [(3, 5), (4, 16), (2, 24), (5, 64), (2, 200), (1, 1000)])
def test_head_norm_with_silu_gate(device, dtype, heads, gs):
    W = heads * gs
    y, w = rand(9, W, seed=1, device=device, dtype=dtype), rand(W, seed=2, device=device)
    gate = rand(9, W + 16, seed=3, device=device, dtype=dtype)[:, 8 : 8 + W]
    out = torch.zeros(9, W + 8, device=device, dtype=dtype)
    ops.head_norm_gate(out[:, :W], y, gate, w, heads, 1e-3)
    n = oracle.unit_rms(f64(y).view(9, heads, gs), 1e-3).reshape(9, W)
    close(out[:, :W], n * f64(w) * oracle.silu(f64(gate)), dtype)
    assert not out[:, W:].any()


@every
def test_norm_of_a_silent_head(device, dtype):
    """eps inside the root: a head of tiny values stays tiny."""
    y = torch.full((2, 16), 1e-4, device=device, dtype=dtype)
    one = torch.ones(16, device=device)
    out = torch.empty_like(y)
    ops.head_norm_gate(out, y, torch.ones_like(y), one, 2, 1e-2)
    want = oracle.unit_rms(f64(y).view(2, 2, 8), 1e-2).view(2, 16) * oracle.silu(
        torch.ones(2, 16).double())
    close(out, want, dtype)
    assert out.abs().max() < 2e-3


# ---------------------------------------------------------------- token shift
@every
@pytest.mark.parametrize("width", [10, 72])
def test_token_shift_over_portions(device, dtype, width):
    """Portions down to one row, several sequences a step, a slot used again."""
    pool = Pool(device, [40, 40, 40])
    mu = rand(5, width, seed=1, device=device)
    h = [rand(40, width, seed=10 + i, device=device, dtype=dtype) for i in range(3)]
    prev = rand(3, width, seed=3, device=device, dtype=dtype)  # left by another sequence

    def want(i):
        x = f64(h[i])
        last = torch.cat([torch.zeros_like(x[:1]), x[:-1]])
        return x + (last - x) * f64(mu)[:, None]

    at = [0, 0, 0]
    for step in ([(0, 1), (1, 7)], [(1, 1), (0, 1), (2, 2)], [(0, 1), (1, 1), (2, 1)],
                 [(2, 3), (0, 20)], [(1, 31), (0, 17), (2, 34)]):
        parts = [(i, at[i], n) for i, n in step]
        b, _ = pool.batch(parts, dtype=dtype)
        x = torch.cat([h[i][s : s + n] for i, s, n in parts])
        got = ops.token_shift(x, mu, prev, b.positions, b.segs)
        for (i, s, n), r in zip(parts, b.segs.cu.tolist()):
            close(got[:, r : r + n], want(i)[:, s : s + n], dtype)
            at[i] = s + n
            assert torch.equal(prev[i], h[i][s + n - 1])
    assert at == [40, 40, 40]


# ------------------------------------------------------------ paged attention
ATTN = [
    # H, G, dim, vdim, cap, block
    (6, 3, 18, 26, 6.0, 16), (4, 4, 16, 24, 30.0, 16), (20, 5, 40, 72, 8.0, 64),
    (18, 1, 136, 16, 50.0, 16), (8, 2, 128, 128, 20.0, 64), (2, 1, 64, 64, 45.0, 32),
    (4, 2, 256, 256, 15.0, 16), (3, 1, 8, 8, 10.0, 8),
]


class Attn:
    def __init__(self, shape, lengths, device, dtype, seed=0):
        self.H, self.G, self.dim, self.vdim, self.cap, block = shape
        self.device, self.dtype, self.pool = device, dtype, Pool(device, lengths, block)
        mk = lambda n, s: [  # noqa: E731
            rand(L, n, seed=seed + 100 * s + i, device=device, dtype=dtype)
            for i, L in enumerate(lengths)
        ]
        self.q, self.k, self.v, self.gate = (
            mk(n, s) for s, n in enumerate(
                (self.H * self.dim, self.G * self.dim, self.G * self.vdim, self.H)))
        self.sink = rand(self.H, seed=seed + 9, device=device)
        self.scale = 2.0 * self.dim ** -0.5
        nb = self.pool.num_blocks
        # what other sequences left in the pages
        self.kp = rand(nb, block, self.G * self.dim, seed=5, device=device, dtype=dtype, mult=30.)
        self.vp = rand(nb, block, self.G * self.vdim, seed=6, device=device, dtype=dtype, mult=30.)

    def want(self, i):
        T = self.q[i].shape[0]
        o = oracle.softmax_attention(
            f64(self.q[i]).view(T, self.H, self.dim), f64(self.k[i]).view(T, self.G, self.dim),
            f64(self.v[i]).view(T, self.G, self.vdim), f64(self.sink), self.scale, self.cap)
        return (o * oracle.sigmoid(f64(self.gate[i]))[..., None] * 0.6).reshape(T, -1)

    def run(self, parts, n_prefill=None):
        """Outputs of the rows of parts [(sequence, start, rows)], in order."""
        b, plan = self.pool.batch(parts, n_prefill, self.dtype)
        pick = lambda xs: torch.cat([xs[i][s : s + n] for i, s, n in parts])  # noqa: E731
        wide = torch.cat([pick(self.q), pick(self.gate)], 1)  # strided operands
        pad = -(self.H * self.dim) % 8
        wide = torch.cat([pick(self.q), pick(self.gate).new_zeros(len(wide), pad),
                          pick(self.gate), wide.new_zeros(len(wide), -self.H % 8)], 1)
        q, at = wide[:, : self.H * self.dim], self.H * self.dim + pad
        ops.page_write(pick(self.k), pick(self.v), self.kp, self.vp, b.slot_mapping)
        out = torch.zeros(len(wide), self.H * self.vdim + 8, dtype=self.dtype, device=self.device)
        ops.paged_attention(
            out[:, : self.H * self.vdim], q, self.kp, self.vp, self.H, self.G, self.sink,
            self.scale, self.cap, wide[:, at : at + self.H], 0.6, b.positions, b.segs, plan)
        assert not out[:, self.H * self.vdim :].any()
        return out[:, : self.H * self.vdim]


@every
@pytest.mark.parametrize("shape", ATTN)
def test_attention_over_schedules(device, dtype, shape):
    """Whole prompts, portions beside single rows, decoding: all sequences."""
    L = [150, 70, 33]
    a = Attn(shape, L, device, dtype)
    want = [a.want(i) for i in range(3)]
    got = a.run([(0, 0, 150), (1, 0, 70), (2, 0, 33)])
    close(got, torch.cat(want), dtype)
    cuts = [([(0, 0, 65), (1, 0, 2)], None), ([(0, 65, 30), (2, 0, 17), (1, 2, 1)], 2),
            ([(0, 95, 15), (1, 3, 60), (2, 17, 1)], 2), ([(0, 110, 1), (1, 63, 1), (2, 18, 1)], 0),
            ([(0, 111, 39), (1, 64, 6), (2, 19, 14)], None)]
    a = Attn(shape, L, device, dtype)
    for parts, n_pre in cuts:
        got = a.run(parts, n_pre)
        close(got, torch.cat([want[i][s : s + n] for i, s, n in parts]), dtype)


@every
@pytest.mark.parametrize("shape", [ATTN[0], ATTN[2], ATTN[4]])
def test_one_key_that_stands_out(device, dtype, shape):
    """A key far back, at page and tile borders, first and last: the row that
    asks for it gets its value, the row before it is there does not."""
    n = 300
    a = Attn(shape, [n], device, dtype, seed=3)
    H, G, dim = a.H, a.G, a.dim
    for at in (0, 1, 15, 16, 31, 32, 63, 64, 127, 128, 255, 256, 298):
        key = rand(dim, seed=at, device=device)
        key = key / key.norm() * dim ** 0.5
        a.k[0][at] = (6.0 * key).repeat(G).to(dtype)
        ask = min(n - 1, at + 171)
        a.q[0][ask] = key.repeat(H).to(dtype)
        if at > 0:
            a.q[0][at - 1] = key.repeat(H).to(dtype)  # not visible yet
        a.v[0][at] = 50.0
    want = a.want(0)
    close(a.run([(0, 0, n)]), want, dtype)
    b = Attn(shape, [n], device, dtype, seed=3)
    b.q, b.k, b.v = a.q, a.k, a.v
    b.run([(0, 0, 120)])
    rows = torch.cat([b.run([(0, t, 1)], 0) for t in range(120, n)])
    close(rows, want[120:], dtype)


@every
def test_the_sink_takes_its_share_once(device, dtype):
    """Equal scores: n keys and a sink of the same score weigh 1/(n+1) each,
    whatever the tiling or split."""
    shape = (4, 2, 16, 16, 20.0, 16)
    n = 600
    a = Attn(shape, [n], device, dtype)
    a.k[0].zero_()
    a.sink.zero_()
    a.gate[0].fill_(20.0)
    a.v[0].fill_(1.0)
    t = torch.arange(n).double()[:, None] + 1
    want = (0.6 * t / (t + 1)).expand(n, 64)
    close(a.run([(0, 0, n)]), want, dtype)
    close(a.run([(0, n - 1, 1)], 0), want[-1:], dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("n", [1, 2, 33, 128, 129, 1000])
def test_decode_splits_of_the_keys(n):
    """One row alone makes several splits; captured shapes do not know n."""
    a = Attn((8, 2, 64, 64, 20.0, 64), [1000], "cuda", BF16)
    a.run([(0, 0, 1000)])
    close(a.run([(0, n - 1, 1)], 0), a.want(0)[n - 1 : n], BF16)


# ------------------------------------------- recurrences, decay per channel
@every
@pytest.mark.parametrize("T,N,R", [(3, 10, 5), (70, 96, 16), (17, 68, 40), (130, 200, 64)])
def test_decay_logs(device, dtype, T, N, R):
    a = rand(T, R + 8, seed=1, device=device, dtype=dtype, mult=2.0)[:, :R]
    w2 = rand(N, R, seed=2, device=device, dtype=dtype, mult=R ** -0.5)
    b = rand(N, seed=3, device=device)
    z = f64(a) @ f64(w2).T + f64(b)
    close(ops.decay_logs(a, w2, b, "sigmoid", 16.0), oracle.log_sigmoid(z) / 16.0, F32, 5)
    z = torch.tanh(f64(a)) @ f64(w2).T + f64(b)
    want = (-torch.exp(z)).clamp(min=-80)  # beyond it, e^log w is as good as 0
    close(ops.decay_logs(a, w2, b, "exp", 1.0).clamp(min=-80), want, F32, 5)


@every
def test_decay_logs_do_not_overflow(device, dtype):
    a = torch.full((2, 8), 100.0, device=device, dtype=dtype)
    w2 = torch.ones(16, 8, device=device, dtype=dtype)
    for kind, b in (("exp", 200.0), ("exp", -200.0), ("sigmoid", -2000.0), ("sigmoid", 200.0)):
        w = ops.decay_logs(a, w2, torch.full((16,), b, device=device), kind, 1.0).exp()
        assert torch.isfinite(w).all() and (w >= 0).all() and (w <= 1).all()
        assert (w < 1e-30).all() if (kind == "exp") == (b > 0) else (w == 1).all()


SIZES = [(3, 14, 22), (2, 72, 72), (2, 136, 200), (4, 64, 64), (1, 24, 300), (2, 256, 64)]


@every
@pytest.mark.parametrize("H,dk,dv", SIZES)
@pytest.mark.parametrize("bonus", [False, True], ids=["gla", "wkv"])
@pytest.mark.parametrize("strength", [0.05, 2.0, 60.0])
def test_recurrence_over_schedules(device, dtype, H, dk, dv, bonus, strength):
    """Whole, in portions around the chunk of 64 rows, token by token, beside
    others; slots that another sequence used; decays near 1 and near 0."""
    L = [150, 97]
    pool = Pool(device, L)
    mk = lambda n, s: [  # noqa: E731
        rand(k, H * n, seed=10 * s + i, device=device, dtype=dtype) for i, k in enumerate(L)]
    q, k, v = mk(dk, 1), mk(dk, 2), mk(dv, 3)
    logw = [-strength * rand(n, H * dk, seed=40 + i, device=device).abs() for i, n in enumerate(L)]
    if strength > 1:
        for w in logw:
            w[10::37] = -75.0  # all but forgotten now and then
    u = rand(H, dk, seed=7, device=device) if bonus else None

    def want(i):
        n = L[i]
        a, b, c = (f64(x[i]).view(n, H, -1) for x in (q, k, v))
        w = torch.exp(f64(logw[i])).view(n, H, dk)
        if bonus:
            return oracle.wkv_recurrence(a * 0.3, b, c, w, f64(u)).reshape(n, -1) \
                if dk == dv else wkv_any(a * 0.3, b, c, w, f64(u)).reshape(n, -1)
        return oracle.gla_recurrence(a * 0.3, b, c, w).reshape(n, -1)

    wants = [want(0), want(1)]
    for cuts in (
        [[(0, 0, 150), (1, 0, 97)]],
        [[(0, 0, 64), (1, 0, 33)], [(1, 33, 2), (0, 64, 63)], [(0, 127, 1), (1, 35, 1)],
         [(0, 128, 22), (1, 36, 61)]],
        [[(0, t, 1)] for t in range(5)] + [[(0, 5, 40), (1, 0, 96)], [(1, 96, 1), (0, 45, 105)]],
    ):
        S = rand(2, H, dv, dk, seed=5, device=device, mult=9.0)  # stale
        for parts in cuts:
            b, plan = pool.batch(parts, dtype=dtype)
            pick = lambda xs: torch.cat([xs[i][s : s + n] for i, s, n in parts])  # noqa: E731
            y = ops.decayed_kv(
                pick(q), pick(k), pick(v), pick(logw), u, 0.3, H, dk, dv, S, b.positions,
                b.segs, plan)
            close(y, torch.cat([wants[i][s : s + n] for i, s, n in parts]), dtype)


def wkv_any(r, k, v, decay, u):
    """oracle.wkv_recurrence with a value size of its own."""
    T, H, d = r.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=r.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out[t] = ((S + u[:, :, None] * kv) * r[t][:, :, None]).sum(1)
        S = decay[t][:, :, None] * S + kv
    return out


@every
def test_state_carries_over_long_decoding(device, dtype):
    """Decays of about 1 - 1e-3: the first token still counts at the end."""
    H, d, n = 2, 16, 300
    pool = Pool(device, [n])
    q = torch.ones(n, H * d, device=device, dtype=dtype)
    k, v = torch.zeros_like(q), torch.zeros_like(q)
    k[0], v[0] = 1.0, 4.0
    logw = torch.full((n, H * d), -1e-3, device=device)
    S = torch.zeros(1, H, d, d, device=device)
    want = d * 4.0 * torch.exp(-1e-3 * torch.arange(n).double())
    for parts in [(0, 0, 100)], *[[(0, t, 1)] for t in range(100, n)]:
        b, plan = pool.batch(parts, dtype=dtype)
        _, s, m = parts[0]
        y = ops.decayed_kv(q[s : s + m], k[s : s + m], v[s : s + m], logw[s : s + m].clone(),
                           None, 1.0, H, d, d, S, b.positions, b.segs, plan)
        close(y, want[s : s + m, None].expand(m, H * d), dtype)


# ------------------------------------------------------------------- experts
@every
@pytest.mark.parametrize("width", [6, 40, 512])
def test_clamped_glu(device, dtype, width):
    x = rand(9, 2 * width, seed=1, device=device, dtype=dtype, mult=3.0)
    g, u = f64(x).split(width, -1)
    g, u = g.clamp(max=1.5), u.clamp(-1.5, 1.5)
    close(ops.clamped_glu(x, 1.5), g * oracle.sigmoid(1.702 * g) * (u + 1), dtype)


def _experts(E, W, ff, device, dtype, seed=0):
    mk = lambda n, k, s: [  # noqa: E731
        rand(n, k, seed=seed + 1000 * s + e, device=device, dtype=dtype, mult=1.5 * k ** -0.5)
        for e in range(E)]
    g, u, d = mk(ff, W, 1), mk(ff, W, 2), mk(W, ff, 3)
    return (g, u, d), ops.pack_experts(ff, W, E, lambda e: (g[e], u[e], d[e]))


def _moe_want(h, z, top, parts, limit, shared):
    g, u, d = parts
    y = f64(shared)
    for t, chosen in enumerate(oracle.route(z, top)):
        for e, p in chosen:
            w = {"gate": f64(g[e]), "up": f64(u[e]), "down": f64(d[e])}
            y[t] = y[t] + p * oracle.clamped_expert(w, f64(h[t]), limit)
    return y


@every
@pytest.mark.parametrize("T,E,top,W,ff", [
    (1, 5, 2, 18, 10), (9, 1, 1, 40, 24), (33, 7, 7, 22, 14), (70, 9, 3, 72, 40),
    (5, 70, 4, 64, 32), (120, 4, 2, 136, 200), (300, 3, 1, 64, 48), (40, 300, 2, 16, 8),
])
def test_experts_and_their_sum(device, dtype, T, E, top, W, ff):
    h = rand(T, W, seed=1, device=device, dtype=dtype)
    wr = rand(E, W, seed=2, device=device, dtype=dtype, mult=2 * W ** -0.5)
    b = rand(E, seed=3, device=device)
    parts, packed = _experts(E, W, ff, device, dtype)
    shared = rand(T, W, seed=4, device=device, dtype=dtype)
    r = ops.route_experts(h, wr, b, top, packed)
    z = f64(h) @ f64(wr).T + f64(b)
    for t, chosen in enumerate(oracle.route(z, top)):  # exact inputs: the same choice
        assert r.ids[t].tolist() == [e for e, _ in chosen]
    close(r.weights, torch.stack([torch.stack([p for _, p in c]) for c in oracle.route(z, top)]),
          F32, 5)
    rows = ops.expert_rows(h, r, packed, 0.8)
    total = ops.ExpertSum(rows, r.slot, r.weights, shared)
    want = _moe_want(h, z, top, parts, 0.8, shared)
    close(total.float(), want, dtype)
    # through the stream kernel, and a selection of rows
    norm = (rand(W, seed=7, device=device), rand(W, seed=8, device=device), 0.9)
    x = rand(T, W, seed=9, device=device)
    y = x.clone()
    ops.add_tanh_norm(y, total, norm, None, dtype)
    d = oracle.dynamic_tanh(want, f64(norm[0]), f64(norm[1]), 0.9)
    close(y, f64(x) + d, dtype)
    idx = torch.tensor([T - 1, 0], device=device)
    y = x[idx].clone()
    ops.add_tanh_norm(y, total[idx], norm, None, dtype)
    close(y, f64(x[idx]) + d[idx.cpu()], dtype)
    if len(want) > 1:  # without a shared expert
        close(ops.ExpertSum(rows, r.slot, r.weights, None).float(), want - f64(shared), dtype, 2)


@every
@pytest.mark.parametrize("T", [3, 50, 700])
def test_all_tokens_to_one_expert(device, dtype, T):
    """The fullest and the emptiest groups, in every form of the products."""
    E, W, ff = 6, 48, 32
    h = rand(T, W, seed=1, device=device, dtype=dtype)
    b = torch.tensor([0.0, 0.0, 0.0, 0.0, 50.0, 0.0], device=device)
    wr = torch.zeros(E, W, device=device, dtype=dtype)
    parts, packed = _experts(E, W, ff, device, dtype)
    r = ops.route_experts(h, wr, b, 1, packed)
    assert (r.ids == 4).all() and (r.weights == 1).all()
    got = ops.ExpertSum(ops.expert_rows(h, r, packed, 1.0), r.slot, r.weights, None).float()
    w = {"gate": f64(parts[0][4]), "up": f64(parts[1][4]), "down": f64(parts[2][4])}
    close(got, oracle.clamped_expert(w, f64(h), 1.0), dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("rows", [16, 32, 64, 256])
def test_every_tile_height_gives_the_same(rows, monkeypatch):
    T, E, W, ff, top = 90, 5, 136, 104, 2
    h = rand(T, W, seed=1, device="cuda", dtype=BF16)
    wr = rand(E, W, seed=2, device="cuda", dtype=BF16)
    b = torch.zeros(E, device="cuda")
    parts, packed = _experts(E, W, ff, "cuda", BF16)
    monkeypatch.setattr(X, "_tile_rows", lambda n, w: rows)
    r = ops.route_experts(h, wr, b, top, packed)
    assert r.tile_rows == rows
    got = ops.ExpertSum(ops.expert_rows(h, r, packed, 1.0), r.slot, r.weights, None).float()
    z = f64(h) @ f64(wr).T
    close(got, _moe_want(h, z, top, parts, 1.0, torch.zeros(T, W)), BF16)


@every
def test_equal_logits_take_the_lower_expert(device, dtype):
    h = torch.ones(4, 16, device=device, dtype=dtype)
    wr = torch.zeros(8, 16, device=device, dtype=dtype)
    _, packed = _experts(8, 16, 8, device, dtype)
    r = ops.route_experts(h, wr, torch.zeros(8, device=device), 3, packed)
    assert r.ids.tolist() == [[0, 1, 2]] * 4
    assert torch.allclose(r.weights, torch.full_like(r.weights, 1 / 3))


def test_experts_are_packed_losslessly():
    """Fragments hold the weights they are made from."""
    w = torch.arange(40 * 24, dtype=torch.float32).view(40, 24)
    f = X._fragments(w)
    assert f.shape == (16, 2, 64, 8)
    for n, k in ((0, 0), (17, 9), (39, 23)):
        lane = n % 16 + 16 * (k % 32 // 8)
        assert f[n // 16, k // 32, lane, k % 8] == w[n, k]
    g, u = torch.ones(20, 4), torch.full((20, 4), 2.0)
    i = X._interleave(g, u)
    assert i.shape[0] == 64 and (i[:16] == 1).all() and (i[16:32] == 2).all()
    assert (i[32:36] == 1).all() and (i[48:52] == 2).all() and not i[36:48].any()
