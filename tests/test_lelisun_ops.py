"""Each mechanism of the hybrid decoders alone, against the float64 oracle:
the CPU ops in fp32, the gfx950 kernels in fp32 and bf16."""

import sys
from pathlib import Path

import numpy as np
import pytest
import torch

sys.path.insert(0, str(Path(__file__).resolve().parent))

import lelisun_oracle as oracle  # noqa: E402
from llmapigateway_amd import ops  # noqa: E402
from llmapigateway_amd.models.batch import ForwardBatch, Segments  # noqa: E402
from llmapigateway_amd.ops import hybrid  # noqa: E402

F32, BF16, F64 = torch.float32, torch.bfloat16, torch.float64
EVERY = [
    pytest.param("cpu", F32, id="cpu-fp32"),
    pytest.param("cuda", F32, id="gpu-fp32", marks=pytest.mark.gpu),
    pytest.param("cuda", BF16, id="gpu-bf16", marks=pytest.mark.gpu),
]
every = pytest.mark.parametrize("device,dtype", EVERY)


def tol(dtype):
    return 1e-2 if dtype == BF16 else 2e-5


def rand(*shape, seed=0, device="cpu", dtype=F32, mult=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * mult).to(dtype).to(device)


def close(got, want, dtype, mult=1.0):
    """Worst row's rms error over the rms of all."""
    got, want = got.double().cpu(), want.double().cpu()
    assert got.shape == want.shape and torch.isfinite(got).all()
    e = (got - want).flatten(1).pow(2).mean(-1).sqrt().max() / want.pow(2).mean().sqrt()
    assert e < tol(dtype) * mult, float(e)


class Pool:
    """Sequences with pages in a scrambled pool and a state slot each."""

    def __init__(self, device, lengths, block=16, slots=None):
        self.device, self.block = device, block
        per = [-(-n // block) for n in lengths]
        g = torch.Generator().manual_seed(7)
        ids = torch.randperm(sum(per) + 3, generator=g)
        self.num_blocks = sum(per) + 3
        self.tables = torch.zeros(len(lengths), max(per), dtype=torch.int32)
        at = 0
        for i, n in enumerate(per):
            self.tables[i, :n] = ids[at : at + n]
            at += n
        self.slots = torch.tensor(slots or range(len(lengths)), dtype=torch.int32)

    def batch(self, parts, n_prefill=None, dtype=F32):
        """parts: [(sequence, start, rows)]; the first n_prefill are prompt
        portions (all by default)."""
        seqs = [p[0] for p in parts]
        starts = np.asarray([p[1] for p in parts], dtype=np.int64)
        lens = np.asarray([p[2] for p in parts], dtype=np.int64)
        n_prefill = len(parts) if n_prefill is None else n_prefill
        cu = np.concatenate([[0], np.cumsum(lens)])
        row_seg = np.repeat(np.arange(len(parts)), lens)
        pos = torch.from_numpy(np.concatenate([np.arange(s, s + n) for s, n in zip(starts, lens)]))
        tables = self.tables[seqs]
        rs = torch.from_numpy(row_seg)
        slot_map = tables[rs, pos // self.block].long() * self.block + pos % self.block
        d = self.device
        segs = Segments(
            cu=torch.tensor(cu, dtype=torch.int32, device=d), slots=self.slots[seqs].to(d),
            tables=tables.to(d), row_seg=rs.int().to(d), block_size=self.block,
            starts=starts, lens=lens, n_prefill=n_prefill,
        )
        b = ForwardBatch(
            kind="prefill" if n_prefill == len(parts) else "mixed",
            token_ids=pos.to(d), positions=pos.to(d), slot_mapping=slot_map.to(d),
            n_prefill_tokens=int(lens[:n_prefill].sum()), segs=segs,
        )
        return b, hybrid.plan_segments(b, dtype)


# ------------------------------------------------------------------ the stream
@every
@pytest.mark.parametrize("width", [7, 96, 1000, 4096, 9000])
def test_stream_add_and_layernorm(device, dtype, width):
    x = rand(5, width, seed=1, device=device, mult=3.0) + 2.0
    d = rand(5, width, seed=2, device=device, dtype=dtype)
    full = rand(5, width, seed=3, device=device)
    vec = rand(width, seed=4, device=device)
    w, b = rand(width, seed=5, device=device), rand(width, seed=6, device=device)
    ref = lambda t: oracle.layer_norm(t.double(), w.double(), b.double(), 1e-3)  # noqa: E731

    y = x.clone()
    close(ops.add_layernorm(y, None, w, b, 1e-3, dtype), ref(x), dtype)
    assert torch.equal(y, x)
    close(ops.add_layernorm(y, d, w, b, 1e-3, dtype), ref(x + d.float()), dtype)
    assert torch.equal(y, x + d.float())
    close(ops.add_layernorm(y, full, w, b, 1e-3, dtype, vec=vec, replace=True),
          ref(full + vec), dtype)
    assert torch.equal(y, full + vec)
    both = torch.zeros(5, 2 * width, dtype=dtype, device=device)
    ops.add_cast(y, d, both[:, :width])
    assert torch.equal(y, full + vec + d.float())
    assert torch.equal(both[:, :width], y.to(dtype)) and not both[:, width:].any()


@every
@pytest.mark.parametrize("width", [7, 128])
def test_scaled_embedding(device, dtype, width):
    e = rand(50, width, seed=1, device=device, dtype=dtype)
    tok = torch.tensor([3, 49, 0, 3], device=device)
    both = torch.zeros(4, 2 * width, dtype=dtype, device=device)
    x = ops.embed_scaled(tok, e, 2.5, both[:, width:])
    assert x.dtype == F32 and torch.equal(x, e[tok].float() * 2.5)
    assert torch.equal(both[:, width:], x.to(dtype)) and not both[:, :width].any()


@every
@pytest.mark.parametrize("T,H,K,N", [(3, 2, 24, 40), (70, 3, 40, 72), (17, 5, 13, 9), (1, 4, 128, 512)])
def test_head_linear(device, dtype, T, H, K, N):
    big = rand(T, H, K + 8, seed=1, device=device, dtype=dtype)
    w = rand(H, N, K, seed=2, device=device, dtype=dtype)
    x = big[..., :K]
    want = torch.stack([x[:, h].double() @ w[h].double().T for h in range(H)], 1)
    close(ops.head_linear(x, w), want, dtype)


@every
@pytest.mark.parametrize("width", [6, 50, 512])
def test_swiglu_any_width(device, dtype, width):
    x = rand(9, 2 * width, seed=1, device=device, dtype=dtype)
    g, u = x.double().split(width, -1)
    close(ops.swiglu(x), oracle.silu(g) * u, dtype)


@every
@pytest.mark.parametrize("groups,width", [(1, 30), (3, 48), (4, 4096), (2, 9000)])
@pytest.mark.parametrize("first", [True, False])
def test_gated_norm(device, dtype, groups, width, first):
    y = rand(4, width, seed=1, device=device, dtype=dtype, mult=0.3)
    both = rand(4, 2 * width, seed=2, device=device, dtype=dtype)
    z, w = both[:, width:], rand(width, seed=3, device=device)
    a, g = y.double(), z.double()
    if first:
        a = a * oracle.silu(g)
    a = oracle.unit_rms(a.view(4, groups, -1), 1e-2).reshape(4, width) * w.double()
    if not first:
        a = a * torch.sigmoid(g)
    close(ops.gated_norm(y, z, w, groups, 1e-2, first), a, dtype)


# ------------------------------------------------------------ latent attention
def latent_pool(pool, rows, rank, rot, dtype):
    """A page pool holding rows[s] [n, rank+rot] of every sequence."""
    width = (rank + rot + 7) // 8 * 8
    cache = torch.zeros(pool.num_blocks, pool.block, width, dtype=dtype)
    cache[..., : rank + rot] = 50.0  # stale rows must not be seen
    flat = cache.view(-1, width)
    for s, r in enumerate(rows):
        p = torch.arange(len(r))
        flat[pool.tables[s, p // pool.block].long() * pool.block + p % pool.block, : rank + rot] = (
            r.to(dtype)
        )
    return cache.to(pool.device)


def attend(q, keys, vals, sink, scale, pos):
    """One row, one head."""
    s = keys[: pos + 1] @ q * scale
    top = torch.maximum(s.max(), sink)
    e = torch.exp(s - top)
    return (e @ vals[: pos + 1]) / (e.sum() + torch.exp(sink - top))


@every
@pytest.mark.parametrize("rank,rot", [(40, 8), (34, 6), (136, 24), (512, 64)])
def test_latent_rows(device, dtype, rank, rot):
    q_rank, T = 56, 19
    pool = Pool(device, [40])
    b, _ = pool.batch([(0, 5, T)])
    d = rand(T, q_rank + rank + rot, seed=1, device=device, dtype=dtype, mult=2.0)
    qn, kn = rand(q_rank, seed=2, device=device), rand(rank, seed=3, device=device)
    cs = ops.build_pair_rope_cache(64, rot, 300.0, device=device)
    width = (rank + rot + 7) // 8 * 8
    cache = torch.zeros(pool.num_blocks, 16, width, dtype=dtype, device=device)
    b.slot_mapping[3] = -1
    cq = ops.latent_rows(d, qn, kn, 1e-2, rot, b.positions, cs, cache, b.slot_mapping)
    dd, pos = d.double().cpu(), b.positions.cpu()
    close(cq, oracle.unit_rms(dd[:, :q_rank], 1e-2) * qn.double().cpu(), dtype)
    c = oracle.unit_rms(dd[:, q_rank : q_rank + rank], 1e-2) * kn.double().cpu()
    kr = oracle.rotate_pairs(dd[:, q_rank + rank :], pos, 300.0, rot)
    keep = [t for t in range(T) if t != 3]
    rows = cache.view(-1, width)[b.slot_mapping[keep]]
    close(rows[:, : rank + rot], torch.cat([c, kr], -1)[keep], dtype)
    assert int((cache.view(-1, width) != 0).any(-1).sum()) == T - 1


@every
@pytest.mark.parametrize("H,dim,rot,rank", [(3, 24, 8, 40), (2, 18, 6, 34), (20, 64, 32, 128)])
def test_fold_queries(device, dtype, H, dim, rot, rank):
    T = 6
    q = rand(T, H, dim + rot, seed=1, device=device, dtype=dtype)
    uk = rand(H, dim, rank, seed=2, device=device, dtype=dtype)
    cs = ops.build_pair_rope_cache(64, rot, 50.0, device=device)
    pos = torch.tensor([0, 1, 2, 17, 40, 63], device=device)
    row = (rank + rot + 7) // 8 * 8
    got = ops.fold_queries(q, uk.transpose(1, 2).contiguous(), row, cs, pos)
    qd = q.double().cpu()
    lat = torch.stack([qd[:, h, :dim] @ uk[h].double().cpu() for h in range(H)], 1)
    close(got[..., :rank], lat, dtype)
    close(got[..., rank : rank + rot],
          oracle.rotate_pairs(qd[..., dim:], pos.cpu(), 50.0, rot), dtype)
    assert not got[..., rank + rot :].any()


@every
@pytest.mark.parametrize("H,rank,rot", [(3, 40, 8), (2, 34, 6), (20, 128, 64), (16, 256, 32), (17, 512, 64)])
def test_folded_attention(device, dtype, H, rank, rot):
    """Random scores, with one key per row that stands out: the first, one
    at a page's or tile's border, the row itself, the one after it (not
    seen)."""
    n = [200, 70, 1]
    pool = Pool(device, n)
    keys = [rand(k, rank + rot, seed=10 + i) for i, k in enumerate(n)]
    probes = [(0, 199, 0), (0, 130, 63), (0, 130, 64), (0, 128, 128), (0, 127, 128), (0, 64, 65),
              (0, 199, 16), (0, 15, 15), (1, 69, 68), (1, 63, 1), (2, 0, 0)]
    row = (rank + rot + 7) // 8 * 8
    q = torch.zeros(len(probes), H, row)
    q[..., : rank + rot] = rand(len(probes), H, rank + rot, seed=3, mult=0.3)
    for t, (s, pos, far) in enumerate(probes):
        q[t, :, : rank + rot] += 0.6 * keys[s][min(far, n[s] - 1)]
    sink = rand(H, seed=4, mult=2.0)
    scale = 12.0 / (rank + rot)
    q = q.to(dtype)
    parts = [(s, pos, 1) for s, pos, _ in probes]
    b, _ = pool.batch(parts, n_prefill=0)
    cache = latent_pool(pool, keys, rank, rot, dtype)
    got = ops.latent_attention_folded(
        q.to(device), cache, rank, sink.to(device), scale, b.positions, b.segs, 0)
    want = torch.empty(len(probes), H, rank, dtype=F64)
    for t, (s, pos, _) in enumerate(probes):
        k = keys[s].to(dtype).double()
        for h in range(H):
            want[t, h] = attend(q[t, h, : rank + rot].double(), k, k[:, :rank], sink[h].double(),
                                scale, pos)
    close(got, want, dtype, mult=1.5)


@pytest.mark.gpu
@pytest.mark.parametrize("H,dim,rot,vdim,rank", [
    (3, 24, 8, 40, 40), (2, 48, 32, 64, 72), (2, 64, 32, 128, 64), (2, 128, 64, 128, 256),
    (3, 200, 24, 152, 64)])
@pytest.mark.parametrize("parts", [
    [(0, 0, 200)], [(0, 0, 50)], [(0, 130, 70), (1, 0, 129), (2, 5, 1)],
    [(1, 60, 9), (0, 64, 136)]])
def test_unfolded_attention(H, dim, rot, vdim, rank, parts):
    """Prompt portions with and without earlier context, keys that stand
    out near and far, against per-head attention."""
    dtype, n = BF16, [200, 129, 6]
    pool = Pool("cuda", n)
    rows = [rand(k, rank + rot, seed=10 + i).to(dtype) for i, k in enumerate(n)]
    cache = latent_pool(pool, rows, rank, rot, dtype)
    wukv = rand(H * (dim + vdim), rank, seed=5, mult=rank ** -0.5).to(dtype)
    sink, scale = rand(H, seed=6, mult=2.0), 0.15
    b, plan = pool.batch(parts, dtype=BF16)
    u = plan.unfold
    if u is None:  # short portions: make the plan all the same
        hybrid.UNFOLD_RATIO, keep = 0, hybrid.UNFOLD_RATIO
        try:
            u = hybrid.plan_segments(b, dtype).unfold
        finally:
            hybrid.UNFOLD_RATIO = keep
    T = b.positions.numel()
    q = rand(T, H, dim + rot, seed=7).to(dtype)
    lat = [r.double()[:, :rank] for r in rows]
    kv = [(x @ wukv.double().T).to(dtype).double() for x in lat]
    pos, seg = b.positions.cpu(), b.segs.row_seg.cpu()
    for t in range(T):  # every third row looks for one key of its past
        if t % 3 == 0:
            s = parts[int(seg[t])][0]
            far = (t * 37) % (int(pos[t]) + 1)
            k = kv[s][far].view(-1)[: H * dim].view(H, dim)
            q[t, :, :dim] += (2.0 * k).to(dtype)
    cs = ops.build_pair_rope_cache(256, rot, 100.0, device="cuda")
    want = torch.empty(T, H, vdim, dtype=F64)
    qd = q.double()
    qr = oracle.rotate_pairs(qd[..., dim:], pos, 100.0, rot).to(dtype).double()
    for t in range(T):
        s = parts[int(seg[t])][0]
        for h in range(H):
            k = torch.cat([kv[s][:, h * dim : (h + 1) * dim], rows[s].double()[:, rank:]], -1)
            v = kv[s][:, H * dim + h * vdim : H * dim + (h + 1) * vdim]
            want[t, h] = attend(torch.cat([qd[t, h, :dim], qr[t, h]]), k, v, sink[h].double(),
                                scale, int(pos[t]))
    got = ops.latent_attention_unfolded(
        q.cuda(), cache, wukv.cuda(), sink.cuda(), scale, dim, vdim, rank, cs, b.positions, u)
    close(got, want, dtype, mult=1.5)


# ----------------------------------------------------------------- recurrences
def cuts(n, sizes):
    """[(start, rows)] that cut n rows by a repeating list of sizes."""
    out, at, k = [], 0, 0
    while at < n:
        m = min(sizes[k % len(sizes)], n - at)
        out.append((at, m))
        at, k = at + m, k + 1
    return out


CUTS = [[131], [1], [2, 3], [64], [65, 1], [31, 32, 33], [100, 1, 1, 29]]


def drive(pool, dtype, lengths, sizes, call):
    """Run every sequence's rows portion by portion, all sequences in a step;
    call(batch, plan, rows) gets the rows as {sequence: slice}."""
    plans = [cuts(n, sizes[i:] + sizes[:i]) for i, n in enumerate(lengths)]
    while any(plans):
        parts = [(i, *p.pop(0)) for i, p in enumerate(plans) if p]
        one = [p for p in parts if p[2] == 1 and p[1] > 0]
        parts = [p for p in parts if p not in one] + one
        b, plan = pool.batch(parts, n_prefill=len(parts) - len(one), dtype=dtype)
        call(b, plan, parts)


@every
@pytest.mark.parametrize("taps", [1, 2, 4, 5])
@pytest.mark.parametrize("C", [11, 48])
def test_causal_conv(device, dtype, taps, C):
    lengths = [131, 40, 3]
    w, bias = rand(C, taps, seed=1), rand(C, seed=2)
    xs = [rand(n, C, seed=3 + i).to(dtype) for i, n in enumerate(lengths)]
    want = [oracle.silu(oracle.causal_conv(x.double(), w.double(), bias.double())) for x in xs]
    wt = w.t().contiguous().to(device)
    for sizes in CUTS:
        pool = Pool(device, lengths, slots=[2, 0, 3])
        state = torch.full((4, taps - 1, C), 9.0, dtype=dtype, device=device)
        got = [torch.zeros(n, C, dtype=F64) for n in lengths]

        def call(b, plan, parts):
            x = torch.cat([xs[i][s : s + n] for i, s, n in parts])
            wide = torch.cat([x, x], -1).to(device)
            y = ops.causal_conv(wide[:, C:], wt, bias.to(device), state, b.positions, b.segs, plan)
            r = 0
            for i, s, n in parts:
                got[i][s : s + n] = y[r : r + n].double().cpu()
                r += n

        drive(pool, dtype, lengths, sizes, call)
        for i in range(3):
            close(got[i], want[i], dtype)
        assert taps == 1 or (state[1] == 9.0).all()  # nobody's slot


@every
@pytest.mark.parametrize("H,P,N,G", [(4, 10, 22, 2), (6, 24, 16, 3), (2, 72, 136, 1), (4, 64, 128, 4)])
def test_ssd(device, dtype, H, P, N, G):
    """Decays from nearly none to nearly all, state carried over portions,
    slots that held another sequence."""
    lengths = [131, 66, 2]
    W = H * P + 2 * G * N
    xs = [rand(n, W, seed=i, mult=0.7).to(dtype) for i, n in enumerate(lengths)]
    dts = [rand(n, H, seed=10 + i, mult=2.0) - 1.0 for i, n in enumerate(lengths)]
    dt_bias, D = rand(H, seed=20, mult=0.3), rand(H, seed=21)
    A_log = torch.linspace(-4.0, 2.0, H)
    want = []
    for x, dt in zip(xs, dts):
        xd = x.double()
        want.append(oracle.mamba2_recurrence(
            xd[:, : H * P].view(-1, H, P), xd[:, H * P : H * P + G * N].view(-1, G, N),
            xd[:, H * P + G * N :].view(-1, G, N), oracle.softplus(dt.double() + dt_bias.double()),
            A_log.double(), D.double()).reshape(-1, H * P))
    c = [t.to(device) for t in (dt_bias, A_log, D)]
    state = torch.full((4, H, P, N), 1e3, device=device)
    for sizes in CUTS:
        pool = Pool(device, lengths, slots=[1, 3, 0])
        got = [torch.zeros(n, H * P, dtype=F64) for n in lengths]

        def call(b, plan, parts):
            x = torch.cat([xs[i][s : s + n] for i, s, n in parts]).to(device)
            dt = torch.cat([dts[i][s : s + n] for i, s, n in parts]).to(device)
            y = ops.ssd(x, dt, *c, H, P, N, G, state, b.positions, b.segs, plan)
            r = 0
            for i, s, n in parts:
                got[i][s : s + n] = y[r : r + n].double().cpu()
                r += n

        drive(pool, dtype, lengths, sizes, call)
        for i in range(3):
            close(got[i], want[i], dtype)
        assert (state[2] == 1e3).all()


@every
@pytest.mark.parametrize("H,dk,dv,cap", [(3, 14, 22, 5.0), (2, 72, 136, 15.0), (2, 16, 200, 8.0), (1, 256, 64, 15.0)])
def test_mlstm(device, dtype, H, dk, dv, cap):
    """Gates over their whole range: input gates near the cap and far below
    it (where the denominator is its floor), forget gates near 0 and 1."""
    lengths = [131, 66, 2]
    qs, ks, vs = ([rand(n, w, seed=j * 10 + i).to(dtype) for i, n in enumerate(lengths)]
                  for j, w in enumerate((H * dk, H * dk, H * dv)))
    gs = []
    for i, n in enumerate(lengths):
        g = rand(n, 2 * H, seed=40 + i, mult=3.0)
        g[:, H:] += 2.0
        g[n // 2 : n // 2 + 9, :H] -= 3 * cap
        g[n // 3 : n // 3 + 2, :H] += 2 * cap
        gs.append(g)
    bias = rand(2 * H, seed=50, mult=0.5)
    want = []
    for q, k, v, g in zip(qs, ks, vs, gs):
        z = cap * torch.tanh((g.double() + bias.double()) / cap)
        want.append(oracle.mlstm_recurrence(
            q.double().view(-1, H, dk) / dk ** 0.5, k.double().view(-1, H, dk),
            v.double().view(-1, H, dv), z[:, :H], oracle.log_sigmoid(z[:, H:])).view(-1, H * dv))
    tiles = -(-dv // 64)
    S = torch.full((4, H, dv, dk), 1e3, device=device)
    n_ = torch.full((4, tiles, H, dk), 1e3, device=device)
    m_ = torch.full((4, tiles, H), 20.0, device=device)
    for sizes in CUTS:
        pool = Pool(device, lengths, slots=[1, 3, 0])
        got = [torch.zeros(n, H * dv, dtype=F64) for n in lengths]

        def call(b, plan, parts):
            def cat(ts):
                return torch.cat([ts[i][s : s + n] for i, s, n in parts]).to(device)
            u = torch.cat([cat(qs), cat(ks), cat(vs)], -1)
            y = ops.mlstm(
                u[:, : H * dk], u[:, H * dk : 2 * H * dk], u[:, 2 * H * dk :], cat(gs),
                bias.to(device), cap, H, dk, dv, S, n_, m_, b.positions, b.segs, plan)
            r = 0
            for i, s, n in parts:
                got[i][s : s + n] = y[r : r + n].double().cpu()
                r += n

        drive(pool, dtype, lengths, sizes, call)
        for i in range(3):
            # rows whose normaliser nearly cancels magnify rounding: compare
            # head by head as the layer does, after the head's own RMS norm
            a = oracle.unit_rms(got[i].view(-1, H, dv), 1e-12).flatten(1)
            w = oracle.unit_rms(want[i].view(-1, H, dv), 1e-12).flatten(1)
            close(a, w, dtype, mult=5.0)
        assert (S[2] == 1e3).all() and (m_[2] == 20.0).all()


@every
def test_padding_rows_touch_no_state(device, dtype):
    """Rows of slot -1 (a captured decode step's padding) leave every state
    as it is and give finite rows."""
    H, P, N, G, C = 2, 16, 24, 1, 2 * 16 + 2 * 24
    pool = Pool(device, [8, 8, 8], slots=[-1, 1, -1])
    b, plan = pool.batch([(0, 3, 1), (1, 3, 1), (2, 0, 1)], n_prefill=0)
    x = rand(3, C, seed=1, device=device, dtype=dtype)
    dt = rand(3, H, seed=2, device=device)
    z = torch.zeros(H, device=device)
    S = rand(3, H, P, N, seed=3, device=device)
    conv = rand(3, 3, C, seed=4, device=device, dtype=dtype)
    S0, c0 = S.clone(), conv.clone()
    y = ops.ssd(x, dt, z, z, z, H, P, N, G, S, b.positions, b.segs, plan)
    u = ops.causal_conv(x, rand(4, C, seed=5, device=device), torch.zeros(C, device=device), conv,
                        b.positions, b.segs, plan)
    for t, t0 in ((S, S0), (conv, c0)):
        assert torch.equal(t[0], t0[0]) and torch.equal(t[2], t0[2])
        assert not torch.equal(t[1], t0[1])
    assert torch.isfinite(y).all() and torch.isfinite(u).all()
