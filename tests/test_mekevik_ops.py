"""Each mechanism of Mekevik alone, against the float64 oracle: the CPU ops in
fp32, the gfx950 kernels in fp32 and bf16."""

import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).resolve().parent))

import mekevik_oracle as oracle  # noqa: E402
from test_lelisun_ops import BF16, F32, Pool, close, every, rand  # noqa: E402
from llmapigateway_amd import ops  # noqa: E402


def f64(t):
    return t.double().cpu()


# ------------------------------------------------------------------ the stream
def _expert_sum(T, W, top, seed, device, dtype):
    rows = rand(T * top + 3, W, seed=seed, device=device, dtype=dtype)
    slot = torch.randperm(T * top + 3, generator=torch.Generator().manual_seed(seed))
    slot = slot[: T * top].view(T, top).int().to(device)
    weights = rand(T, top, seed=seed + 1, device=device).abs()
    want = (f64(rows)[slot.long().cpu()] * f64(weights)[..., None]).sum(1)
    return ops.ExpertSum(rows, slot, weights, None), want


@every
@pytest.mark.parametrize("width", [7, 96, 1000, 4096, 16384])
def test_stream_adds_and_rms_norms(device, dtype, width):
    x = rand(5, width, seed=1, device=device, mult=2.0)
    w1, w2 = rand(width, seed=2, device=device), rand(width, seed=3, device=device)
    d1 = rand(5, width, seed=4, device=device, dtype=dtype)
    d2 = rand(5, width, seed=5, device=device, dtype=dtype)
    experts, ew = _expert_sum(5, width, 3, 6, device, dtype)
    y = x.clone()
    (got,) = ops.add_rms_norm(y, (), (w1,), 1e-3, dtype)
    close(got, oracle.rms_norm(f64(x), f64(w1), 1e-3), dtype)
    assert torch.equal(x, y)
    for deltas, add in (((d1,), f64(d1)), ((d1, d2), f64(d1) + f64(d2)), ((experts,), ew),
                        ((d1, experts), f64(d1) + ew)):
        y = x.clone()
        a, b = ops.add_rms_norm(y, deltas, (w1, w2), 1e-3, dtype)
        stream = f64(x) + add
        close(y, stream, F32, 5)
        close(a, oracle.rms_norm(stream, f64(w1), 1e-3), dtype)
        close(b, oracle.rms_norm(stream, f64(w2), 1e-3), dtype)


@every
def test_epsilon_is_inside_the_root(device, dtype):
    x = torch.full((2, 64), 1e-3, device=device)
    (got,) = ops.add_rms_norm(x, (), (torch.ones(64, device=device),), 1e-2, dtype)
    close(got, oracle.rms_norm(f64(x), 1.0, 1e-2), dtype)
    assert got.abs().max() < 0.02


@every
@pytest.mark.parametrize("wq,wk,wv", [(30, 10, 14), (96, 32, 48), (4096, 1024, 1024)])
@pytest.mark.parametrize("blend", [None, 0.3])
def test_query_key_norms_value_blend_and_pages(device, dtype, wq, wk, wv, blend):
    pool = Pool(device, [9, 5])
    b, _ = pool.batch([(0, 0, 9), (1, 0, 5)], dtype=dtype)
    T, pad = 14, -(wq + wk) % 8
    u = rand(T, wq + wk + pad + wv, seed=1, device=device, dtype=dtype, mult=3.0)
    q, k, v = u[:, :wq], u[:, wq : wq + wk], u[:, wq + wk + pad :]
    qn, kn = rand(wq, seed=2, device=device), rand(wk, seed=3, device=device)
    first = rand(T, wv + 8, seed=4, device=device, dtype=dtype)[:, :wv]
    kp = torch.full((pool.num_blocks, 16, wk), 7.0, device=device, dtype=dtype)
    vp = torch.full((pool.num_blocks, 16, wv), 7.0, device=device, dtype=dtype)
    slots = b.slot_mapping.clone()
    slots[3] = -1  # a row that is not kept
    got = ops.qkv_rows(q, k, v, qn, kn, 1e-2, blend or 0.0, None if blend is None else first,
                       kp, vp, slots)
    close(got, oracle.rms_norm(f64(q), f64(qn), 1e-2), dtype)
    want_v = f64(v) if blend is None else (1 - blend) * f64(v) + blend * f64(first)
    keep = [i for i in range(T) if i != 3]
    at = slots[keep]
    close(kp.view(-1, wk)[at], oracle.rms_norm(f64(k), f64(kn), 1e-2)[keep], dtype)
    close(vp.view(-1, wv)[at], want_v[keep], dtype)
    if blend is None:
        assert torch.equal(vp.view(-1, wv)[at], v[keep])
    rest = torch.ones(kp.shape[0] * 16, dtype=torch.bool)
    rest[at.cpu()] = False
    assert (kp.view(-1, wk)[rest.to(device)] == 7).all()


# ------------------------------------------------------------- distance biases
@pytest.mark.parametrize("rows,far", [
    (32, 128), (32, 128.5), (16, 256), (8, 9), (24, 1000), (2, 2), (3, 17), (64, 33), (32, 4096),
])
@pytest.mark.parametrize("window", [1, 5, 40, 5000])
def test_distance_table(rows, far, window):
    rel, pb = rand(rows, 3, seed=1), rand(3, seed=2)
    t = ops.distance_bias(rel, pb, far, window)
    assert t.shape[1] == 16 and not t[:, 3:].any() and t.shape[0] <= min(window, far + 2)
    for n in range(min(window, 4200)):
        want = rel[oracle.bucket(n, rows, far)] + pb
        assert torch.equal(t[min(n, t.shape[0] - 1), :3], want), n


def test_distances_on_a_boundary_take_the_upper_row():
    """Where ln(n / half) / ln(far / half) is a whole number of rows exactly,
    the floor is that number."""
    t = ops.distance_bias(torch.arange(9.0)[:, None], torch.zeros(1), 128, 1000)[:, 0]
    # rows 4 .. 8, a factor of 2 each: distances 4, 8, 16, 32, 64
    assert [int(t[n]) for n in (3, 4, 7, 8, 15, 16, 31, 32, 63, 64, 128)] == [
        3, 4, 4, 5, 5, 6, 6, 7, 7, 8, 8]


# ---------------------------------------------------------- sigmoid attention
ATTN = [
    # H, G, dim, vdim, window, bias_max, table rows, page
    (6, 3, 18, 26, 37, 21, 10, 16), (8, 2, 40, 64, 50, 40, 16, 16),
    (16, 4, 72, 32, 33, 90, 24, 64), (24, 8, 16, 16, 64, 33, 8, 32),
    (32, 8, 128, 128, 100, 64, 32, 64), (40, 2, 24, 64, 1000, 256, 32, 16),
    (64, 4, 128, 72, 60, 30, 12, 16), (4, 4, 256, 256, 45, 40, 8, 16),
    (20, 5, 200, 24, 70, 16, 6, 16), (1, 1, 8, 8, 1, 4, 4, 16), (12, 4, 64, 40, 90, 300, 20, 16),
    (24, 4, 128, 112, 31, 50, 10, 16), (3, 1, 8, 8, 20, 30, 6, 8),
]


class Attn:
    def __init__(self, shape, lengths, device, dtype, seed=0, pb=-1.0):
        self.H, self.G, self.dim, self.vdim, self.window, self.far, rows, block = shape
        H, G = self.H, self.G
        self.device, self.dtype, self.pool = device, dtype, Pool(device, lengths, block)
        mk = lambda n, s: [  # noqa: E731
            rand(L, n, seed=seed + 100 * s + i, device=device, dtype=dtype)
            for i, L in enumerate(lengths)
        ]
        self.q, self.k, self.v, self.gate = (
            mk(n, s) for s, n in enumerate((H * self.dim, G * self.dim, G * self.vdim,
                                            H * self.vdim)))
        self.rel, self.pb = rand(rows, H, seed=seed + 7), rand(H, seed=seed + 8) + pb
        self.talk = (torch.eye(H) + rand(H, H, seed=seed + 9, mult=H ** -0.5)).to(BF16)
        self.scale = 2.0 * self.dim ** -0.5
        nb = self.pool.num_blocks
        # what other sequences left in the pages
        self.kp = rand(nb, block, G * self.dim, seed=5, device=device, dtype=dtype, mult=30.)
        self.vp = rand(nb, block, G * self.vdim, seed=6, device=device, dtype=dtype, mult=30.)

    def want(self, i):
        T = self.q[i].shape[0]
        w = oracle.attention_weights(
            f64(self.q[i]).view(T, self.H, self.dim), f64(self.k[i]).view(T, self.G, self.dim),
            self.scale, f64(self.rel), self.far, f64(self.pb), self.window)
        o = oracle.apply_weights(
            oracle.mix_heads(w, f64(self.talk)), f64(self.v[i]).view(T, self.G, self.vdim))
        return o.reshape(T, -1) * oracle.sigmoid(f64(self.gate[i]))

    def run(self, parts, n_prefill=None):
        """Outputs of the rows of parts [(sequence, start, rows)], in order."""
        b, plan = self.pool.batch(parts, n_prefill, self.dtype)
        pick = lambda xs: torch.cat([xs[i][s : s + n] for i, s, n in parts])  # noqa: E731
        ops.page_write(pick(self.k), pick(self.v), self.kp, self.vp, b.slot_mapping)
        n_out = self.H * self.vdim
        q, gate = pick(self.q), pick(self.gate)
        wide = torch.cat([q, q.new_zeros(len(q), 8 + -q.shape[1] % 8), gate], 1)  # strided
        out = torch.zeros(len(q), n_out + 8, dtype=self.dtype, device=self.device)
        bias = ops.distance_bias(self.rel.to(self.device), self.pb.to(self.device), self.far,
                                 self.window)
        ops.sigmoid_attention(
            out[:, :n_out], wide[:, : q.shape[1]], self.kp, self.vp, self.H, self.G, self.scale,
            bias, self.talk.to(self.device, self.dtype), self.window, wide[:, -n_out:],
            b.positions, b.segs, plan)
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
    close(got, torch.cat(want), dtype, 2)
    cuts = [([(0, 0, 65), (1, 0, 2)], None), ([(0, 65, 30), (2, 0, 17), (1, 2, 1)], 2),
            ([(0, 95, 15), (1, 3, 60), (2, 17, 1)], 2), ([(0, 110, 1), (1, 63, 1), (2, 18, 1)], 0),
            ([(0, 111, 39), (1, 64, 6), (2, 19, 14)], None)]
    a = Attn(shape, L, device, dtype)
    for parts, n_pre in cuts:
        got = a.run(parts, n_pre)
        close(got, torch.cat([want[i][s : s + n] for i, s, n in parts]), dtype, 2)


@every
@pytest.mark.parametrize("H,G,dim,vdim", [(6, 3, 18, 26), (8, 2, 40, 64), (32, 8, 128, 128)])
@pytest.mark.parametrize("window", [1, 16, 33, 64, 100])
def test_window_and_page_edges(device, dtype, H, G, dim, vdim, window):
    """All weights are near 0 but those of one key, which everybody looks for:
    the last row that sees it gets its value, the next one does not; nor do
    the rows before it."""
    n = 260
    a = Attn((H, G, dim, vdim, window, 50, 16, 16), [n], device, dtype, seed=3, pb=-18.0)
    a.rel.zero_()
    key = rand(dim, seed=1, device=device)
    key = (key / key.norm() * dim ** 0.5).to(dtype)
    a.k[0].zero_()
    a.q[0][:] = key.repeat(H)
    for at in (0, 15, 48, 127, 140):
        a.k[0].zero_()
        a.k[0][at] = 12.0 * key.repeat(G)
        want = a.want(0)
        size = want.abs().amax(-1)
        sees = torch.zeros(n, dtype=torch.bool)
        sees[at : at + window] = True
        assert (size[sees] > 100 * size[~sees].max()).all()
        got = a.run([(0, 0, n)])
        close(got[sees.to(device)], want[sees], dtype, 2)
        assert ((got.abs().amax(-1).cpu() > 1e-2) == sees).all()
        # alone, the pages around it being full (of later tokens, too)
        for t in (at - 1, at, at + window - 1, at + window):
            if 0 <= t < n:
                got = a.run([(0, t, 1)], 0)
                assert (got.abs().max() > 1e-2) == bool(sees[t])
                if sees[t]:
                    close(got, want[t : t + 1], dtype, 2)


@every
def test_weights_are_not_normalized(device, dtype):
    """n keys of equal score weigh the same each, whatever n."""
    a = Attn((4, 2, 16, 16, 200, 20, 8, 16), [300], device, dtype)
    a.rel.zero_(), a.pb.zero_()
    a.k[0].zero_(), a.v[0].fill_(0.125), a.gate[0].zero_()
    a.talk = torch.eye(4).to(BF16)
    t = torch.arange(300).double()[:, None].clamp(max=199) + 1
    want = (0.5 * 0.5 * 0.125 * t).expand(300, 64)
    close(a.run([(0, 0, 300)]), want, dtype)
    close(a.run([(0, 299, 1)], 0), want[-1:], dtype)


@every
@pytest.mark.parametrize("H,G", [(8, 2), (16, 4), (32, 8), (24, 8), (48, 16), (5, 5)])
def test_every_head_reads_the_weights_it_should(device, dtype, H, G):
    """Head h only looks at key h + 3; head h then takes head 7h + 2's weights
    to its own key head's values."""
    n, dim = 90, 64
    a = Attn((H, G, dim, 8, 200, 20, 8, 16), [n], device, dtype, pb=-30.0)
    a.rel.zero_(), a.pb.fill_(-30.0)
    q = torch.nn.functional.normalize(rand(H, dim, seed=1), dim=-1)
    if H <= dim:  # orthogonal directions, one a head
        q = torch.linalg.qr(rand(dim, dim, seed=1).double()).Q[:H].float()
    a.q[0][:] = (8.0 * q).reshape(-1).to(device, dtype)
    a.k[0].zero_()
    for h in range(H):
        g = h // (H // G)
        a.k[0][h + 3, g * dim : (g + 1) * dim] = (60.0 * q[h]).to(device, dtype)
    perm = [(7 * h + 2) % H for h in range(H)]
    a.talk = torch.zeros(H, H).to(BF16)
    for h, other in enumerate(perm):
        a.talk[h, other] = 1.0
    a.gate[0].fill_(30.0)
    rows = a.run([(0, 0, n)])
    last = rows[-1].view(H, 8).cpu()
    v = a.v[0].view(n, G, 8).cpu()
    for h, other in enumerate(perm):
        assert torch.allclose(last[h].float(), v[other + 3, h // (H // G)].float(),
                              atol=0.02, rtol=0.02), h
    close(rows, a.want(0), dtype)
    close(a.run([(0, n - 1, 1)], 0)[0].view(H, 8), last, dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("n", [1, 2, 31, 32, 33, 128, 129, 1000, 2500])
@pytest.mark.parametrize("window", [40, 700, 5000])
def test_decode_splits_of_the_keys(n, window):
    """One row alone makes several splits; captured shapes do not know n."""
    a = Attn((8, 2, 64, 64, window, 128, 32, 64), [n + 1], "cuda", BF16, pb=-3.0)
    b, _ = a.pool.batch([(0, 0, n)], dtype=BF16)
    ops.page_write(a.k[0][:n], a.v[0][:n], a.kp, a.vp, b.slot_mapping)
    T = n + 1  # the oracle's last row alone
    lo = max(0, T - window)
    k, v = f64(a.k[0]).view(T, 2, 64)[lo:], f64(a.v[0]).view(T, 2, 64)[lo:]
    s = torch.einsum("hd,nhd->hn", f64(a.q[0][n]).view(8, 64), k.repeat_interleave(4, 1))
    rows = [oracle.bucket(T - 1 - j, 32, 128) for j in range(lo, T)]
    w = oracle.sigmoid(s * a.scale + f64(a.rel)[rows].T + f64(a.pb)[:, None])
    o = torch.einsum("hn,nhd->hd", f64(a.talk) @ w, v.repeat_interleave(4, 1)).reshape(1, -1)
    close(a.run([(0, n, 1)], 0), o * oracle.sigmoid(f64(a.gate[0][n:])), BF16)


@pytest.mark.gpu
def test_many_steps_of_a_wave():
    """More than 32 steps of 128 keys in one split: page lists are reloaded."""
    n = 5000
    a = Attn((2, 1, 16, 16, 6000, 128, 32, 16), [n], "cuda", BF16, pb=-4.0)
    b, _ = a.pool.batch([(0, 0, n)], dtype=BF16)
    ops.page_write(a.k[0], a.v[0], a.kp, a.vp, b.slot_mapping)
    rows = torch.arange(n - 300, n, device="cuda", dtype=torch.int64)
    want = a.run([(0, n - 300, 300)])  # tiles
    from llmapigateway_amd.ops import hybrid

    batch, _ = a.pool.batch([(0, n - 300, 300)], dtype=BF16)
    bias = ops.distance_bias(a.rel.cuda(), a.pb.cuda(), a.far, a.window)
    out = torch.empty(300, 32, dtype=BF16, device="cuda")
    ops.sigmoid_attention(  # 300 rows: one split each
        out, a.q[0][rows], a.kp, a.vp, 2, 1, a.scale, bias, a.talk.cuda(), a.window,
        a.gate[0][rows].contiguous(), batch.positions, batch.segs, hybrid.SegmentPlan())
    close(out, want, BF16)


# -------------------------------------------------------------------- experts
@every
@pytest.mark.parametrize("T,E,top,W,ff", [
    (1, 5, 2, 18, 10), (33, 7, 7, 22, 14), (70, 9, 3, 72, 40), (120, 4, 2, 136, 200),
    (300, 3, 1, 64, 48), (40, 300, 2, 16, 8),
])
def test_silu_experts_and_their_scaled_weights(device, dtype, T, E, top, W, ff):
    h = rand(T, W, seed=1, device=device, dtype=dtype)
    wr = rand(E, W, seed=2, device=device, dtype=dtype, mult=2 * W ** -0.5)
    mk = lambda n, k, s: [  # noqa: E731
        rand(n, k, seed=1000 * s + e, device=device, dtype=dtype, mult=1.5 * k ** -0.5)
        for e in range(E)]
    g, u, d = mk(ff, W, 1), mk(ff, W, 2), mk(W, ff, 3)
    packed = ops.pack_experts(ff, W, E, lambda e: (g[e], u[e], d[e]))
    r = ops.route_experts(h, wr, None, top, packed, 1.7)
    chosen = oracle.route(f64(h) @ f64(wr).T, top, 1.7)
    assert r.ids.tolist() == [[e for e, _ in c] for c in chosen]
    close(r.weights, torch.stack([torch.stack([p for _, p in c]) for c in chosen]), F32, 5)
    total = ops.ExpertSum(ops.expert_rows(h, r, packed, None), r.slot, r.weights, None)
    want = torch.zeros(T, W).double()
    for t, c in enumerate(chosen):
        for e, p in c:
            w = {"gate": f64(g[e]), "up": f64(u[e]), "down": f64(d[e])}
            want[t] += p * oracle.silu_expert(w, f64(h[t]))
    close(total.float(), want, dtype)
