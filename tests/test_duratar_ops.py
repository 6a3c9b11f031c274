"""Each mechanism of Duratar alone, against the float64 oracle: the CPU ops in
fp32, the gfx950 kernels in fp32 and bf16."""

import math
import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).resolve().parent))

import duratar_oracle as oracle  # noqa: E402
from lelisun_oracle import unit_rms  # noqa: E402
from test_lelisun_ops import BF16, F32, Pool, close, every, rand  # noqa: E402
from llmapigateway_amd import ops  # noqa: E402
from llmapigateway_amd.models.streams import DEFER, HyperStreams  # noqa: E402


def f64(t):
    return t.double().cpu()


# ------------------------------------------------------------------ the stream
@every
@pytest.mark.parametrize("width", [7, 96, 1000, 4096, 16384])
def test_embedding_norm(device, dtype, width):
    embed = rand(30, width, seed=1, device=device, dtype=dtype, mult=0.3)
    w, toks = rand(width, seed=2, device=device), torch.tensor([3, 29, 0, 3], device=device)
    got = ops.embed_rms_norm(toks, embed, w, 1e-2)
    close(got, unit_rms(f64(embed[toks]), 1e-2) * f64(w), F32)


@every
@pytest.mark.parametrize("S", [1, 2, 3, 4, 5, 8, 11, 16])
@pytest.mark.parametrize("width", [70, 128, 2048])
def test_streams_over_many_sublayers(device, dtype, S, width):
    """Reads and rewrites at their own times, against all streams kept."""
    T, subs = 5, 11
    mk = lambda *s, seed: rand(*s, seed=seed)  # noqa: E731
    coefs = [(mk(S, seed=3 * q), torch.eye(S) + 0.4 * mk(S, S, seed=3 * q + 1),
              1.0 + 0.3 * mk(S, seed=3 * q + 2)) for q in range(subs)]
    hs = HyperStreams(S, coefs, device)
    assert sum(r.rewrite for r in hs.reads) == (subs - 1) // DEFER and len(hs.reads) == subs + 1
    e = rand(T, width, seed=100, device=device)
    x, pending = e.clone().unsqueeze(1), []
    streams = torch.stack([f64(e)] * S)
    for q, (w_in, mix, w_out) in enumerate(coefs):
        norm = rand(width, seed=200 + q, device=device)
        h, x, pending = hs.read(q, x, pending, norm, 1e-3, dtype)
        want = oracle.read_streams(streams, w_in.double())
        close(h, unit_rms(want, 1e-3) * f64(norm), dtype, 2)
        y = rand(T, width, seed=300 + q, device=device, dtype=dtype)
        scale = None if q == 2 else rand(width, seed=400 + q, device=device)
        pending = pending + [(y, scale)]
        streams = oracle.write_streams(streams, mix.double(), w_out.double(),
                                       f64(y) * (1.0 if scale is None else f64(scale)))
    norm, pick = rand(width, seed=500, device=device), torch.tensor([4, 1], device=device)
    h, _, _ = hs.read(subs, x, pending, norm, 1e-3, dtype, pick)
    close(h, (unit_rms(streams.sum(0), 1e-3) * f64(norm))[[4, 1]], dtype, 2)


def test_streams_are_mixed_from_the_old_ones():
    """mix is [from, to]; every new stream takes the old ones."""
    mix, out = torch.tensor([[0.0, 1.0], [0.0, 0.0]]), torch.tensor([0.0, 1.0])
    first, second = torch.tensor([1.0, 0.0]), torch.tensor([0.0, 1.0])
    hs = HyperStreams(2, [(w, mix, out) for w in (first, first, second)], "cpu")
    e, pending = torch.arange(1.0, 9.0).view(1, 1, 8), []
    x = e
    # y = 5: x2 = e + 5, x1 = 0; y = 7: x2 = 0 + 7
    for q, want in enumerate((e[0], torch.zeros(1, 8), torch.full((1, 8), 7.0))):
        h, x, pending = hs.read(q, x, pending, torch.ones(8), 1.0, F32)
        assert torch.allclose(h, unit_rms(want, 1.0))
        pending = pending + [(torch.full((1, 8), 5.0 + 2.0 * q), None)]


@every
@pytest.mark.parametrize("n", [1, 7, 96, 4096])
def test_xielu(device, dtype, n):
    z = rand(9, n, seed=1, device=device, dtype=dtype, mult=3.0)
    z[0] *= 1e-3
    z[1, 0] = 0.0
    z[2] -= 30.0
    p, q = torch.tensor(0.3).double(), torch.tensor(-1.2).double()
    want = oracle.xielu(f64(z), p, q)
    small = oracle.xielu(f64(z[0]), p, q)
    sp = lambda v: math.log1p(math.exp(v))  # noqa: E731
    got = ops.xielu_(z, sp(0.3), 0.5 + sp(-1.2))
    assert got is z
    close(z, want, dtype)
    close(z[:1], small[None], dtype)


# ------------------------------------------------------------- rotary q and k
SCALING = {"factor": 3.0, "low": 1.5, "high": 3.0, "original": 200}


@pytest.mark.parametrize("dims,base", [(2, 50.0), (16, 1e4), (64, 5e5)])
@pytest.mark.parametrize("scaling", [None, SCALING, dict(SCALING, low=1.0, high=8.0)])
def test_rotary_table(dims, base, scaling):
    """All three kinds of frequencies: kept, divided, in between."""
    t = ops.build_pair_rope_cache(301, dims, base, scaling=scaling)
    f = oracle.frequencies({"dims": dims, "base": base, "scaling": scaling})
    ang = torch.arange(301).double()[:, None] * torch.tensor(f, dtype=torch.float64)
    assert torch.allclose(t, torch.cat([ang.cos(), ang.sin()], -1).float(), atol=1e-6, rtol=0)
    if scaling and dims > 2:
        plain = oracle.frequencies({"dims": dims, "base": base})
        kinds = {"kept" if a == b else "cut" if abs(a * scaling["factor"] - b) < 1e-12 else "mid"
                 for a, b in zip(f, plain)}
        assert kinds >= {"kept", "cut"}


def test_rotary_wavelength_edges():
    """At low and high themselves both formulas agree; just beyond they hold."""
    for turns, want in ((3.0, 1.0), (3.0001, 1.0), (1.5, 1 / 3), (1.4999, 1 / 3), (2.25, 2 / 3)):
        f = turns * 2 * math.pi / 200
        got = oracle.frequencies({"dims": 2, "base": 1.0, "scaling": dict(
            SCALING, original=200 * f)})[0]
        assert abs(got - want) < 1e-3
        t = ops.build_pair_rope_cache(2, 2, 1.0, scaling=dict(SCALING, original=200 * f))
        assert abs(math.atan2(t[1, 1], t[1, 0]) - got) < 1e-6


@every
@pytest.mark.parametrize("nq,nk,dim,rot,wv", [
    (6, 2, 18, 6, 10), (6, 3, 18, 18, 7), (8, 2, 24, 16, 40), (12, 4, 64, 32, 128),
    (4, 4, 128, 128, 72), (2, 2, 256, 16, 256), (5, 1, 40, 0, 8), (3, 1, 70, 32, 1000),
    (8, 2, 72, 24, 64),
])
def test_rotary_rows(device, dtype, nq, nk, dim, rot, wv):
    pool = Pool(device, [9, 5])
    b, _ = pool.batch([(0, 0, 9), (1, 0, 5)], dtype=dtype)
    T = 14
    mk = lambda n: -(-n // 8) * 8  # noqa: E731
    wq, wk = nq * dim, nk * dim
    u = rand(T, mk(wq) + mk(wk) + wv + 8, seed=1, device=device, dtype=dtype, mult=2.0)
    q, k = u[:, :wq], u[:, mk(wq) : mk(wq) + wk]
    v = u[:, mk(wq) + mk(wk) : mk(wq) + mk(wk) + wv]
    qn, kn = rand(dim, seed=2, device=device), rand(dim, seed=3, device=device)
    cs = ops.build_pair_rope_cache(16, rot, 300.0, device=device, scaling=SCALING)
    kp = torch.full((pool.num_blocks, 16, wk), 7.0, device=device, dtype=dtype)
    vp = torch.full((pool.num_blocks, 16, wv), 7.0, device=device, dtype=dtype)
    slots = b.slot_mapping.clone()
    slots[3] = -1  # a row that is not kept
    got = ops.rotary_rows(q, k, v, qn, kn, 1e-2, cs, b.positions, kp, vp, slots)

    def want(x, w):
        x = unit_rms(f64(x).view(T, -1, dim), 1e-2) * f64(w)
        cfg = {"dims": rot, "base": 300.0, "scaling": SCALING}
        return torch.cat([oracle.rotate_half(p, cfg) for p in (x[:9], x[9:])]).view(T, -1)

    close(got, want(q, qn), dtype)
    keep = [i for i in range(T) if i != 3]
    at = slots[keep]
    close(kp.view(-1, wk)[at], want(k, kn)[keep], dtype)
    assert torch.equal(vp.view(-1, wv)[at], v[keep])
    rest = torch.ones(kp.shape[0] * 16, dtype=torch.bool)
    rest[at.cpu()] = False
    assert (kp.view(-1, wk)[rest.to(device)] == 7).all()
    assert (vp.view(-1, wv)[rest.to(device)] == 7).all()
    alone = ops.rotary_rows(q, None, None, qn, None, 1e-2, cs, b.positions, kp, vp, slots)
    assert torch.equal(alone, got)


# ------------------------------------------------------------ window attention
ATTN = [
    # H, G, maps, dim, vdim, window, kept, page
    (6, 3, 2, 18, 26, 37, 5, 16), (4, 1, 2, 32, 64, 50, 3, 16), (8, 2, 2, 40, 72, 33, 40, 64),
    (8, 8, 2, 64, 128, 64, 1, 32), (6, 1, 2, 128, 136, 100, 17, 64), (24, 2, 2, 16, 24, 45, 7, 16),
    (2, 2, 2, 96, 200, 31, 70, 16), (4, 2, 2, 24, 16, 1, 2, 16), (3, 3, 2, 8, 8, 20, 0, 8),
    (8, 2, 1, 40, 64, 50, 6, 16), (20, 1, 1, 128, 128, 90, 33, 64), (2, 1, 1, 200, 256, 40, 3, 16),
    (4, 4, 1, 10, 12, 1000, 0, 16), (32, 2, 1, 64, 40, 65, 64, 32), (16, 4, 2, 64, 64, 128, 16, 64),
]


class Attn:
    def __init__(self, shape, lengths, device, dtype, seed=0, mult=2.0):
        self.H, self.G, self.maps, self.dim, self.vdim, self.window, self.keep, block = shape
        H, G, M = self.H, self.G, self.maps
        self.device, self.dtype, self.pool = device, dtype, Pool(device, lengths, block)
        mk = lambda n, s: [  # noqa: E731
            rand(L, n, seed=seed + 100 * s + i, device=device, dtype=dtype)
            for i, L in enumerate(lengths)
        ]
        self.q, self.k, self.v = (
            mk(n, s) for s, n in enumerate((H * M * self.dim, G * M * self.dim, G * self.vdim)))
        self.scale, self.lam, self.diff, self.eps = mult * self.dim ** -0.5, 0.7, 0.4, 1e-3
        nb = self.pool.num_blocks
        # what other sequences left in the pages
        self.kp = rand(nb, block, G * M * self.dim, seed=5, device=device, dtype=dtype, mult=30.)
        self.vp = rand(nb, block, G * self.vdim, seed=6, device=device, dtype=dtype, mult=30.)

    def want(self, i, raw=False):
        T, H, G, M = self.q[i].shape[0], self.H, self.G, self.maps
        q, k = f64(self.q[i]).view(T, H, M, -1), f64(self.k[i]).view(T, G, M, -1)
        v, seen, out = f64(self.v[i]).view(T, G, -1), oracle.visible(T, self.window, self.keep), []
        for h in range(H):
            g = h // (H // G)
            a = [oracle.softmax_map(q[:, h, m], k[:, g, m], v[:, g], self.scale, seen)
                 for m in range(M)]
            out.append(a[0] if M == 1 else oracle.combine_maps(
                *a, self.lam, self.diff, self.eps))
        return torch.cat(out, -1)

    def run(self, parts, n_prefill=None):
        """Outputs of the rows of parts [(sequence, start, rows)], in order."""
        b, plan = self.pool.batch(parts, n_prefill, self.dtype)
        pick = lambda xs: torch.cat([xs[i][s : s + n] for i, s, n in parts])  # noqa: E731
        ops.page_write(pick(self.k), pick(self.v), self.kp, self.vp, b.slot_mapping)
        n_out, q = self.H * self.vdim, pick(self.q)
        wide = torch.cat([q, q.new_zeros(len(q), 8 + -q.shape[1] % 8)], 1)  # strided
        out = torch.zeros(len(q), n_out + 8, dtype=self.dtype, device=self.device)
        ops.window_attention(
            out[:, :n_out], wide[:, : q.shape[1]], self.kp, self.vp, self.H, self.G, self.maps,
            self.scale, self.window, self.keep, self.lam, 1.0 - self.diff, self.eps, b.positions,
            b.segs, plan)
        assert not out[:, n_out:].any()
        return out[:, :n_out]


@every
@pytest.mark.parametrize("shape", ATTN)
def test_attention_over_schedules(device, dtype, shape):
    """Whole prompts, portions beside single rows, decoding: all sequences."""
    L = [150, 70, 33]
    a = Attn(shape, L, device, dtype)
    want = [a.want(i) for i in range(3)]
    got = a.run([(0, 0, 150), (1, 0, 70), (2, 0, 33)])
    close(got, torch.cat(want), dtype, 3)
    cuts = [([(0, 0, 65), (1, 0, 2)], None), ([(0, 65, 30), (2, 0, 17), (1, 2, 1)], 2),
            ([(0, 95, 15), (1, 3, 60), (2, 17, 1)], 2), ([(0, 110, 1), (1, 63, 1), (2, 18, 1)], 0),
            ([(0, 111, 39), (1, 64, 6), (2, 19, 14)], None)]
    a = Attn(shape, L, device, dtype)
    for parts, n_pre in cuts:
        got = a.run(parts, n_pre)
        close(got, torch.cat([want[i][s : s + n] for i, s, n in parts]), dtype, 3)


@every
@pytest.mark.parametrize("H,G,maps,dim,vdim", [
    (6, 3, 2, 18, 26), (4, 2, 2, 40, 64), (4, 1, 2, 64, 128), (8, 2, 1, 32, 40)])
@pytest.mark.parametrize("window,keep", [(1, 0), (16, 1), (33, 16), (64, 17), (100, 70)])
def test_window_kept_and_page_edges(device, dtype, H, G, maps, dim, vdim, window, keep):
    """Everybody looks for one key: the rows that see it get its value, no
    other row does; at the edges of pages, of the window and of the kept ones."""
    n = 260
    a = Attn((H, G, maps, dim, vdim, window, keep, 16), [n], device, dtype, seed=3)
    key = rand(dim, seed=1, device=device)
    key = (key / key.norm() * dim ** 0.5).to(dtype)
    a.q[0][:] = key.repeat(H * maps)
    mark = (rand(a.vdim, seed=2, device=device).sign() * 3.0).to(dtype).repeat(G)
    a.lam = 0.25  # the maps agree: what is left keeps its sign
    for at in {0, 15, 127, 140, max(keep - 1, 0), keep, 2 * keep + 16}:
        a.k[0].zero_(), a.v[0].normal_(generator=torch.Generator(device).manual_seed(at))
        a.k[0][at] = 30.0 * key.repeat(G * maps)
        a.v[0][at] = mark
        want = a.want(0)
        t = torch.arange(n)
        sees = (t >= at) & ((t - at < window) | torch.tensor(at < keep))
        match = (want * f64(mark.repeat_interleave(1).view(G, vdim).repeat_interleave(
            H // G, 0).reshape(-1)).sign()[None]).mean(-1)
        if window > 1:
            assert match[sees].min() > 2 * match[~sees].abs().max() if (~sees).any() else True
        close(a.run([(0, 0, n)]), want, dtype, 3)
        # alone, the pages around it being full (of later tokens, too)
        for p in (at - 1, at, at + window - 1, at + window, n - 1):
            if 0 <= p < n:
                close(a.run([(0, p, 1)], 0), want[p : p + 1], dtype, 3)


@every
def test_maps_and_heads_read_their_own_keys(device, dtype):
    """Head h's map m only looks at key 2h + m + 3."""
    H, G, dim, vdim, n = 8, 2, 32, 16, 60
    a = Attn((H, G, 2, dim, vdim, 200, 0, 16), [n], device, dtype, mult=1.0)
    q = torch.linalg.qr(rand(dim, dim, seed=1).double()).Q[: 2 * H].float()
    a.q[0][:] = (10.0 * q).reshape(-1).to(device, dtype)
    a.k[0].zero_()
    kv = a.k[0].view(n, G, 2, dim)
    for h in range(H):
        for m in range(2):
            kv[2 * h + m + 3, h // (H // G), m] += (30.0 * q[2 * h + m]).to(device, dtype)
    for rows in (a.run([(0, 0, n)])[-1], a.run([(0, n - 1, 1)], 0)[0]):
        got, v = f64(rows).view(H, vdim), f64(a.v[0]).view(n, G, vdim)
        for h in range(H):
            g = h // (H // G)
            o = oracle.combine_maps(v[2 * h + 3, g], v[2 * h + 4, g], a.lam, a.diff, a.eps)
            assert (got[h] - o).abs().max() < 0.03, h


@pytest.mark.gpu
@pytest.mark.parametrize("n", [0, 1, 2, 31, 32, 33, 128, 129, 1000, 2500])
@pytest.mark.parametrize("window,keep", [(40, 3), (700, 130), (5000, 0)])
def test_decode_splits_of_the_keys(n, window, keep):
    """One row alone makes several splits; captured shapes do not know n."""
    a = Attn((8, 2, 2, 64, 64, window, keep, 64), [n + 1], "cuda", BF16)
    if n:
        b, _ = a.pool.batch([(0, 0, n)], dtype=BF16)
        ops.page_write(a.k[0][:n], a.v[0][:n], a.kp, a.vp, b.slot_mapping)
    close(a.run([(0, n, 1)], 0), a.want(0)[n:], BF16, 3)


# ----------------------------------------------------------------- recurrences
SCHEDULES = [
    [([(0, 0, 150), (1, 0, 70), (2, 0, 33)], None)],
    [([(0, 0, 65), (1, 0, 2)], None), ([(0, 65, 30), (2, 0, 17), (1, 2, 1)], 2),
     ([(0, 95, 15), (1, 3, 60), (2, 17, 1)], 2), ([(0, 110, 1), (1, 63, 1), (2, 18, 1)], 0),
     ([(0, 111, 39), (1, 64, 6), (2, 19, 14)], None)],
    [([(0, 0, 1), (1, 0, 1), (2, 0, 1)], 0)] + [
        ([(0, t, 1), (1, t, 1), (2, t, 1)], 0) for t in range(1, 20)
    ] + [([(0, 20, 130), (1, 20, 50), (2, 20, 13)], None)],
]
L = [150, 70, 33]


def over_schedules(dtype, device, want, step, state):
    """step(batch, plan, pick, state) of every schedule against want[i]; state
    slots hold what other sequences left."""
    for schedule in SCHEDULES:
        pool, S = Pool(device, L, slots=[2, 0, 1]), state.clone()
        for parts, n_pre in schedule:
            b, plan = pool.batch(parts, n_pre, dtype)
            pick = lambda xs: torch.cat([xs[i][s : s + n] for i, s, n in parts])  # noqa: E731
            got = step(b, plan, pick, S)
            close(got, torch.cat([want[i][s : s + n] for i, s, n in parts]), dtype, 2)


@every
@pytest.mark.parametrize("H,dk,dv", [
    (3, 18, 26), (2, 16, 40), (4, 64, 64), (2, 128, 136), (1, 200, 72), (1, 300, 16)])
@pytest.mark.parametrize("decays", [(0.9, 0.999), (0.5, 1.0), (0.0, 0.02)])
def test_fixed_decays(device, dtype, H, dk, dv, decays):
    decay = [decays[h % 2] for h in range(H)]
    wide = 2 * (-(-H * dk // 8) * 8)
    us = [rand(n, wide + H * dv + 8, seed=i, device=device, dtype=dtype, mult=1.5)
          for i, n in enumerate(L)]
    cut = lambda u: (u[:, : H * dk], u[:, wide // 2 : wide // 2 + H * dk],  # noqa: E731
                     u[:, wide : wide + H * dv])
    want = []
    for u in us:
        q, k, v = (oracle.silu(f64(x)).view(len(u), H, -1) for x in cut(u))
        want.append(oracle.lightning_recurrence(q, k, v, decay).reshape(len(u), -1))

    def step(b, plan, pick, S):
        return ops.fixed_decay_kv(
            *cut(pick(us)), torch.tensor(decay, device=device), H, dk, dv, S, b.positions, b.segs,
            plan)

    over_schedules(dtype, device, want, step, rand(3, H, dv, dk, seed=9, device=device, mult=50.))


@every
@pytest.mark.parametrize("T,N,R", [(1, 18, 5), (70, 40, 8), (130, 264, 24), (5, 128, 200)])
def test_softplus_decays(device, dtype, T, N, R):
    a = rand(T, R + 8, seed=1, device=device, dtype=dtype)[:, :R]
    w2 = rand(N, R, seed=2, device=device, dtype=dtype, mult=2 * R ** -0.5)
    bias, A_log = rand(N, seed=3, device=device) - 2.0, rand(2, seed=4)
    rate = A_log.exp().repeat_interleave(N // 2).to(device)
    got = ops.decay_logs(a, w2, bias, "softplus", rate=rate)
    assert got.dtype == F32
    want = oracle.channel_decay(f64(a), f64(w2), f64(bias), f64(A_log), 2).log().view(T, N)
    close(got, want.clamp(min=-80), F32, 10)


def _delta_case(H, G, dk, dv, device, dtype, spread):
    wide = -(-G * dk // 8) * 8
    xs = [rand(n, 2 * wide + H * dv, seed=i, device=device, dtype=dtype) for i, n in enumerate(L)]
    bs = [rand(n, H + 8, seed=20 + i, device=device, dtype=dtype, mult=2.) for i, n in enumerate(L)]
    logs = [-spread * torch.exp(rand(n, H * dk, seed=30 + i, device=device)) for i, n in enumerate(L)]
    cut = lambda x: (x[:, : G * dk], x[:, wide : wide + G * dk], x[:, 2 * wide :])  # noqa: E731
    want = []
    for x, b, w in zip(xs, bs, logs):
        q, k, v = (f64(t) for t in cut(x))
        q, k = (oracle.unit_vectors(t.view(len(x), G, dk)).repeat_interleave(H // G, 1)
                for t in (q, k))
        want.append(oracle.delta_recurrence(
            q * dk ** -0.5, k, v.view(len(x), H, dv), torch.exp(f64(w)).view(len(x), H, dk),
            oracle.sigmoid(f64(b[:, :H]))).reshape(len(x), -1))

    def step(batch, plan, pick, S):
        return ops.delta_kv(*cut(pick(xs)), pick(logs), pick(bs)[:, :H], H, G, dk, dv, S,
                            batch.positions, batch.segs, plan)

    return xs, bs, want, step


@every
@pytest.mark.parametrize("H,G,dk,dv", [
    (3, 3, 18, 26), (4, 2, 16, 40), (2, 2, 64, 64), (4, 1, 72, 16), (2, 1, 128, 136),
    (1, 1, 200, 72), (1, 1, 300, 16), (2, 2, 24, 200)])
@pytest.mark.parametrize("spread", [0.02, 0.5, 6.0])
def test_delta_rule(device, dtype, H, G, dk, dv, spread):
    """Weak, middling and strong decays: the last ones leave the range in which
    a block's products factor."""
    _, _, want, step = _delta_case(H, G, dk, dv, device, dtype, spread)
    over_schedules(dtype, device, want, step, rand(3, H, dv, dk, seed=9, device=device, mult=50.))


@every
def test_delta_rule_replaces_what_a_key_holds(device, dtype):
    """beta near 1 and no decay: writing a key again replaces its value, at
    any distance, across chunks and portions; the read-out sees the write."""
    H, dk, dv, n = 2, 64, 64, 150
    keys = torch.linalg.qr(rand(dk, dk, seed=1).double()).Q[:10].float()
    at = torch.randint(0, 10, (n,), generator=torch.Generator().manual_seed(3))
    k = (4.0 * keys[at]).repeat(1, H).to(device, dtype)
    v = rand(n, H * dv, seed=2, device=device, dtype=dtype)
    b = torch.full((n, H), 20.0, device=device, dtype=dtype)
    for sizes in ([150], [70, 1, 79], [1] * 40 + [110]):
        pool, S, t = Pool(device, [n]), rand(1, H, dv, dk, seed=4, device=device), 0
        for m in sizes:
            bt, plan = pool.batch([(0, t, m)], 1 if m > 1 else 0, dtype)
            q = k[(torch.arange(t, t + m) - 3).clamp(min=0)]  # what was written 3 rows ago
            logw = torch.zeros(m, H * dk, device=device)
            s = slice(t, t + m)
            y = ops.delta_kv(q, k[s], v[s], logw, b[s], H, H, dk, dv, S, bt.positions, bt.segs, plan)
            for i in range(m):
                a = int(at[max(t + i - 3, 0)])
                last = max(j for j in range(t + i + 1) if int(at[j]) == a)
                assert (y[i] * dk ** 0.5 - v[last]).abs().max() < (0.15 if dtype == BF16 else 1e-3)
            t += m


@every
@pytest.mark.parametrize("heads,gs", [(3, 18), (4, 64), (2, 520)])
def test_head_norm_with_a_sigmoid_gate(device, dtype, heads, gs):
    T, W = 6, heads * gs
    y = rand(T, W, seed=1, device=device, dtype=dtype)
    gate = rand(T, W + 8, seed=2, device=device, dtype=dtype)[:, :W]
    w, out = rand(gs, seed=3, device=device).repeat(heads), torch.empty_like(y)
    ops.head_norm_gate(out, y, gate, w, heads, 1e-2, act="sigmoid")
    want = unit_rms(f64(y).view(T, heads, gs), 1e-2).view(T, W) * f64(w)
    close(out, want * oracle.sigmoid(f64(gate)), dtype)


@every
@pytest.mark.parametrize("taps", [1, 2, 4, 6])
def test_convolution_without_a_bias(device, dtype, taps):
    C = 40
    xs = [rand(n, C, seed=i, device=device, dtype=dtype) for i, n in enumerate(L)]
    w = rand(C, taps, seed=9)
    want = [oracle.causal_conv(f64(x), w.double()) for x in xs]

    def step(b, plan, pick, S):
        return ops.causal_conv(pick(xs), w.t().contiguous().to(device),
                               torch.zeros(C, device=device), S, b.positions, b.segs, plan)

    over_schedules(dtype, device, want, step,
                   rand(3, taps - 1, C, seed=8, device=device, dtype=dtype, mult=50.))
