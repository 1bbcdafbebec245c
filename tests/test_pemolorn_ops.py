"""Each mechanism of the Pemolorn decoder alone, against the plain implementation."""
import math

import numpy as np
import pytest
import torch

import pemolorn_oracle as oracle
from copilot_for_consensus_amd.models.projection import Projection
from copilot_for_consensus_amd.ops import branch as N
from copilot_for_consensus_amd.ops import gqa as A
from copilot_for_consensus_amd.ops import gru as R
from copilot_for_consensus_amd.ops import moe as M
from copilot_for_consensus_amd.ops import stream as S
from copilot_for_consensus_amd.ops.cols import Cols
from copilot_for_consensus_amd.ops.reference import moe_rows
from copilot_for_consensus_amd.runtime.kv_cache import PagedHeads

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]


def rnd(*shape, seed=0, scale=1.0):
    return scale * torch.randn(*shape, generator=torch.Generator().manual_seed(seed + 31 * len(shape) + sum(shape)))


def close(got, want, tol):
    got, want = got.float().cpu(), want.float()
    assert torch.isfinite(got).all()
    assert float((got - want).abs().max()) <= tol * max(1.0, float(want.abs().max())), float((got - want).abs().max())


def tol(dtype):
    return 2e-5 if dtype == torch.float32 else 1.2e-2


def i32(x, device="cpu"):
    return torch.tensor(np.asarray(x), dtype=torch.int32, device=device)


def slabs(x, n, seed=7):
    """fp32 parts whose sum is x."""
    parts = rnd(n, *x.shape, seed=seed)
    parts[-1] = x - parts[:-1].sum(0)
    return parts


# ------------------------------------------------------------------ branches between two norms
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,T,split", [(104, 5, 1), (65, 3, 3), (1500, 4, 9), (5000, 2, 2), (4096, 3, 4)])
@pytest.mark.parametrize("kind", ["none", "one", "two", "routed"])
def test_branch_and_norms(device, dtype, W, T, split, kind):
    x, eps, g, n = 3 * rnd(T, W), 1e-2, rnd(1, seed=1), rnd(1 if split % 2 else W, seed=2)
    d = lambda t: t.to(device).contiguous()
    y, z, w1, w2 = rnd(T, W, seed=3), 0.1 * rnd(T, W, seed=4), rnd(W, seed=5), rnd(W, seed=6)
    br, want = None, x
    if kind == "one":
        br, total = N.Branch(d(g), eps, y=d(slabs(y, split))), y
    elif kind == "two":
        br = N.Branch(d(g), eps, y=d(slabs(y, split)), w=d(w1), y2=d(slabs(z, 2)), w2=d(w2))
        total = (oracle.rms(y, eps) * w1 + oracle.rms(z, eps) * w2) / 2
    elif kind == "routed":
        top, experts = 1 + split, 5
        rows, own = rnd(3 * T, W, seed=7).to(dtype), rnd(T, W, seed=8).to(dtype)
        pos = torch.randint(0, 3 * T, (T, top), generator=torch.Generator().manual_seed(0))
        ids = torch.randint(0, experts + 3, (T, top), generator=torch.Generator().manual_seed(1))
        ids[0] = experts                                     # a token that chooses nothing but itself
        wt = rnd(T, top, seed=9)
        br = N.Branch(d(g), eps, routed=(d(rows), i32(pos, device), d(wt), i32(ids, device), experts, d(own)))
        pick = [[own[t] if ids[t, c] >= experts else rows[pos[t, c]] for c in range(top)] for t in range(T)]
        total = torch.stack([sum(wt[t, c] * pick[t][c].float() for c in range(top)) for t in range(T)])
    if br is not None:
        want = x + oracle.scalar_norm(total, g, eps)
    xg, h = d(x).clone(), torch.empty(T, W, dtype=dtype, device=device)
    N.branch_norm(xg, br, d(n), eps, h)
    close(xg, want, 3e-5)
    close(h, oracle.rms(want, eps) * n, tol(dtype))
    if br is not None and kind != "routed":
        xg = d(x).clone()
        N.branch_norm(xg, br, None, eps, None)
        close(xg, want, 3e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,F,split", [(3, 65, 1), (5, 256, 3), (2, 1030, 11)])
def test_squared_relu(device, dtype, T, F, split):
    x = rnd(T, F)
    close(S.relu_sq(slabs(x, split).to(device), dtype), torch.clamp(x, min=0.0) ** 2, tol(dtype))


@pytest.mark.gpu
@pytest.mark.parametrize("M,N,K", [(300, 24704, 128), (1, 192, 64), (513, 25600, 192), (100, 256, 320), (6200, 1024, 192)])
def test_squared_relu_of_a_product(M, N, K):
    """Every kernel a product takes, among them the prompt product's epilogue with whole and cut tiles."""
    x, w = rnd(M, K).to(torch.bfloat16), rnd(N, K, seed=1, scale=K ** -0.5).to(torch.bfloat16)
    got = Projection(w.cuda()).relu_sq(x.cuda())
    close(got, torch.clamp(x.float() @ w.float().T, min=0.0) ** 2, 8e-3)


# ------------------------------------------------------------------ recurrence
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [1, 33, 96, 1024, 260])
def test_recurrence_in_portions_and_decoded(device, dtype, W):
    """Whole, in portions down to one token that carry the state, and token by token: other slots untouched."""
    T = 203
    z, u, g = (rnd(T, W, seed=s, scale=2.0).to(dtype).float() for s in (1, 2, 3))
    bz, bx = rnd(W, seed=4) - 2.0, rnd(W, seed=5)
    want = oracle.min_gru((z + bz).double(), (u + bx).double()).float()
    want = want * g * torch.sigmoid(g)
    p = R.Gru(bz.to(device), bx.to(device))
    zug = torch.cat([z, u, g], 1).to(device, dtype)
    for cuts in ([203], [64, 1, 2, 63, 65, 8], [1, 1, 130, 71]):
        state = rnd(4, W, seed=6).to(device)                 # stale values: a first token does not read them
        before, at = state.clone(), 0
        for n in cuts:
            c = [Cols(zug[at:at + n], k * W, W) for k in range(3)]
            ch, cu = R.chunk_plan([0, n])
            out = R.prefill(p, *c, i32([2], device), i32([0, n], device), i32([at + n], device), i32(ch, device), i32(cu, device),
                            state, torch.empty(n, W, dtype=dtype, device=device))
            close(out, want[at:at + n], tol(dtype))
            at += n
        assert torch.equal(state[[0, 1, 3]], before[[0, 1, 3]])
        last = state[2].clone()
    state = rnd(4, W, seed=7).to(device)
    parts = torch.stack([slabs(torch.cat([z[t:t + 1], u[t:t + 1], g[t:t + 1]], 1), 3, seed=t) for t in range(20)]).to(device)
    for t in range(20):
        c = [Cols(parts[t], k * W, W) for k in range(3)]
        out = R.step(p, *c, i32([1], device), i32([t + 1], device), state, torch.empty(1, W, dtype=dtype, device=device))
        close(out, want[t:t + 1], tol(dtype))
    # a batch: portions of several sequences in one launch
    lens, slots = [70, 1, 130], [3, 0, 2]
    state, cu = rnd(4, W, seed=8).to(device), np.cumsum([0] + lens).tolist()
    idx = torch.cat([torch.arange(n) for n in lens])
    c = [Cols(zug[idx.to(device)], k * W, W) for k in range(3)]
    ch, ccu = R.chunk_plan(cu)
    out = R.prefill(p, *c, i32(slots, device), i32(cu, device), i32(lens, device), i32(ch, device), i32(ccu, device), state,
                    torch.empty(cu[-1], W, dtype=dtype, device=device))
    close(out, want[idx], tol(dtype))
    assert last.shape == (W,)


# ------------------------------------------------------------------ projections to queries and cache rows
def heads_of(H, G, dim, vdim, per_head, conv, rot, mask, seed=0, device="cpu", shared=False, sink=True):
    nq, nk, nv = H * dim, G * dim, G * vdim
    w = rnd(conv, nq + nk + nv, seed=seed + 1) if conv else None
    qn, kn = rnd(dim if per_head else nq, seed=seed + 2), rnd(dim if per_head else nk, seed=seed + 3)
    return A.Heads(H, G, dim, vdim, 0.3, mask, 1e-3, qn.to(device), kn.to(device), per_head, rnd(H, seed=seed + 4).to(device) if sink else None,
                   A.rope_freq(rot, 500.0, device), w.to(device) if conv else None, shared)


def want_qkv(a, u, T0=0):
    """The plain q, k, v [T, heads, .] of projections u [T, columns]."""
    T, nq, nk = u.shape[0], a.H * a.dim, a.G * a.dim
    if a.conv is not None:
        u = oracle.short_conv(u, a.conv.cpu().T)
    pos, rot = torch.arange(T), 0 if a.freq is None else 2 * a.freq.numel()

    def turned(x, w, n):
        w = w.cpu()
        x = oracle.rms(x.view(T, n, a.dim), a.eps) * w if a.per_head else (oracle.rms(x, a.eps) * w).view(T, n, a.dim)
        return oracle.rotate(x, pos, 500.0, rot) if rot else x
    q = turned(u[:, :nq], a.q_norm, a.H)
    if a.shared:
        return q, None, None
    return q, turned(u[:, nq:nq + nk], a.k_norm, a.G), u[:, nq + nk:].view(T, a.G, a.vdim)


def gather(cache, table, n):
    """Rows 0 .. n - 1 of a sequence [n, G, D] from [blocks, G, entries, D]."""
    e = cache.shape[2]
    return torch.stack([cache[table[i // e], :, i % e] for i in range(n)]).float().cpu()


QKV = [  # H, G, dim, vdim, per head, taps, rot, pool, split (0: activations)
    (4, 2, 64, 64, True, 0, 0, 0, 0), (4, 2, 32, 48, False, 4, 32, 8, 0), (3, 1, 18, 14, False, 3, 6, 5, 0),
    (2, 2, 36, 9, True, 0, 0, 0, 2), (6, 3, 24, 40, False, 7, 10, 3, 3), (8, 2, 128, 128, False, 4, 64, 16, 5),
    (1, 1, 7, 5, False, 1, 2, 1, 1), (40, 8, 128, 128, True, 0, 0, 0, 0), (2, 1, 300, 16, True, 2, 150, 40, 0), (2, 1, 80, 80, True, 0, 16, 0, 1)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", QKV)
def test_projections_to_cache_rows(device, dtype, case):
    """Convolution, norms, rotation, cache rows and pooled means: portions of every kind, then decoded tokens, on scattered
    pages and a used state slot."""
    H, G, dim, vdim, per_head, taps, rot, pool, split = case
    mask = A.Mask(20, pool=pool) if pool else A.Mask(20, keep=2)
    a = heads_of(H, G, dim, vdim, per_head, taps, rot, mask, device=device)
    T, C, e = 90, a.columns, A.pool_entries(pool) if pool else 0
    u = rnd(T, C, seed=11).to(dtype).float()
    q, k, v = want_qkv(a, u)
    rows = PagedHeads(8, G, a.D, pool, e, device, dtype)
    tail = rnd(3, max(taps - 1, 0), C, seed=12).to(device) if taps > 1 else None
    table = [5, 2, 7]
    bt, at, got = i32([table], device), 0, []
    for n in [37, 2, 1, 3, 27] + [1] * 20:
        pos = i32(range(at, at + n), device)
        slots = i32([table[p // 32] * 32 + p % 32 for p in range(at, at + n)], device)
        part = u[at:at + n]
        cols = Cols(slabs(part, split).to(device) if split else part.to(device, dtype))
        decoded = n == 1 and at > 60
        if decoded:
            got.append(A.qkv_rows(a, cols, rows, pos, slots, i32([1], device), bt, tail))
        else:
            got.append(A.qkv_rows(a, cols, rows, pos, slots, i32([1] * n, device), bt, tail, i32(range(n), device)))
            A.conv_tail(a, cols, i32([0, n], device), i32([at + n], device), i32([1], device), tail)
            if pool:
                A.pool_rows(a, rows, i32(A.ended_blocks([0, n], [at + n], pool), device), bt)
        at += n
    got = torch.cat(got).float().cpu()
    close(got[..., :dim], q * 0.3 * A.LOG2E, tol(dtype))
    assert not got[..., dim:].any()
    close(gather(rows.k, table, T)[..., :dim], k, tol(dtype))
    close(gather(rows.v, table, T)[..., :vdim], v, tol(dtype))
    assert not gather(rows.k, table, T)[..., dim:].any() and not rows.k[[0, 1, 3, 4, 6]].any()
    if pool:
        n = T // pool
        # means of what the cache holds
        close(gather(rows.pk, table, n), oracle.pooled(gather(rows.k, table, T), pool), 2e-6 if dtype == torch.float32 else 4e-3)
        close(gather(rows.pv, table, n), oracle.pooled(gather(rows.v, table, T), pool), 2e-6 if dtype == torch.float32 else 4e-3)


@pytest.mark.parametrize("device", DEVICES)
def test_queries_alone_leave_the_cache(device):
    a = heads_of(4, 2, 32, 32, True, 0, 0, A.Mask(9, keep=2), device=device, shared=True)
    rows = PagedHeads(2, 2, a.D, 0, 0, device, torch.float32)
    u = rnd(5, a.columns, seed=3)
    q = A.qkv_rows(a, Cols(u.to(device)), rows, i32(range(5), device), i32(range(5), device), None, i32([[0]], device), None, i32(range(5), device))
    close(q, want_qkv(a, u)[0] * 0.3 * A.LOG2E, 2e-5)
    assert not rows.k.any() and not rows.v.any()


def test_pooled_entries_lie_on_pages_that_exist():
    for pool in range(1, 70):
        e = A.pool_entries(pool)
        assert e & (e - 1) == 0 and e * pool >= 32
        for b in range(200):
            assert b // e <= (b * pool + pool - 1) // 32
    assert A.ended_blocks([0, 5, 6, 30], [5, 17, 40], 8).tolist() == [[2, 2], [2, 3], [2, 4]]
    assert A.ended_blocks([0, 1, 9], [16, 8], 8).tolist() == [[0, 1], [1, 0]]


# ------------------------------------------------------------------ attention
ATTN = [  # H, G, dim, vdim, size, keep, pool
    (4, 2, 64, 64, 40, 3, 0), (4, 2, 96, 96, 33, 0, 8), (3, 1, 18, 14, 17, 0, 5), (2, 2, 36, 9, 64, 70, 0), (20, 1, 128, 128, 100, 5, 0),
    (8, 2, 128, 100, 63, 0, 16), (40, 1, 32, 32, 1, 1, 0), (2, 1, 140, 160, 31, 0, 1), (2, 1, 192, 180, 65, 0, 33), (1, 1, 256, 256, 50, 20, 0),
    (2, 2, 300, 33, 45, 0, 7), (4, 4, 64, 64, 0, 0, 0), (4, 1, 64, 61, 500, 0, 4), (2, 1, 128, 128, 64, 0, 64), (2, 1, 64, 64, 5, 0, 100)]


def attn_case(case, T, dtype, device, seed=0, sink=True):
    """A sequence's q, k, v (k and v rounded) in a cache of scattered pages, with its pooled means."""
    H, G, dim, vdim, size, keep, pool = case
    a = heads_of(H, G, dim, vdim, True, 0, 0, A.Mask(size, keep, pool), seed, device, sink=sink)
    q, k, v = rnd(T, H, dim, seed=seed + 21), rnd(T, G, dim, seed=seed + 22), rnd(T, G, vdim, seed=seed + 23)
    return a, q, k, v


def fill(a, rows, k, v, table, device):
    T = k.shape[0]
    for i in range(T):
        rows.k[table[i // 32], :, i % 32, :a.dim] = k[i].to(rows.k.dtype).to(device)
        rows.v[table[i // 32], :, i % 32, :a.vdim] = v[i].to(rows.v.dtype).to(device)
    if a.mask.pool:
        A.pool_rows(a, rows, i32([[0, b] for b in range(T // a.mask.pool)] or np.zeros((0, 2)), device), i32([table], device))


def want_attn(a, q, k, v, dtype, rounded=True):
    m = {"size": a.mask.size or 10 ** 6, "keep_first": a.mask.keep} | ({"pool": a.mask.pool} if a.mask.pool else {})
    k, v = (t.to(dtype).float() for t in (k, v))
    sink = a.sink.cpu() if a.sink is not None else torch.full((a.H,), -1e30)
    return oracle.attend((q * a.scale * A.LOG2E).to(dtype).float() / A.LOG2E, k, v, 1.0, m, sink)


def packed_q(a, q, dtype, device):
    out = torch.zeros(q.shape[0], a.H, a.D, dtype=dtype, device=device)
    out[..., :a.dim] = (q * a.scale * A.LOG2E).to(dtype).to(device)
    return out


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", ATTN)
def test_attention_in_portions_and_decoded(device, dtype, case):
    """Two sequences at once: a whole prompt, portions at page, tile and window edges, and single tokens in one and in
    several key slices; a garbage page in the pool does not matter."""
    lens, tables = [300, 131], [[3, 9, 1, 14, 7, 5, 11, 0, 8, 2], [13, 4, 6, 12, 10]]
    seqs = [attn_case(case, n, dtype, device, seed=100 * i) for i, n in enumerate(lens)]
    a = seqs[0][0]
    e = A.pool_entries(a.mask.pool) if a.mask.pool else 0
    rows = PagedHeads(16, a.G, a.D, a.mask.pool, e, device, dtype)
    for t in rows.tensors():
        t.normal_(0.0, 3.0)                                 # what other sequences left
    for t, w in ((rows.k, a.dim), (rows.v, a.vdim)):
        t[..., w:] = 0.0
    for (_, _, k, v), table in zip(seqs, tables):
        fill(a, rows, k, v, table, device)
    want = [want_attn(a, q, k, v, dtype) for _, q, k, v in seqs]
    width = max(map(len, tables))
    full = [t + [0] * (width - len(t)) for t in tables]
    limit = 3e-5 if dtype == torch.float32 else 1.5e-2
    n_rows = A.prompt_rows(dtype, a.D)
    for cuts in ([(0, 300), (0, 131)], [(63, 66), (0, 2)], [(64, 129), (31, 33)], [(299, 300), (40, 131)], [(33, 290), (128, 131)]):
        q = torch.cat([s[1][lo:hi] for s, (lo, hi) in zip(seqs, cuts)])
        cu, ctx = np.cumsum([0] + [hi - lo for lo, hi in cuts]).tolist(), [hi for _, hi in cuts]
        got = A.attention(a, packed_q(a, q, dtype, device), rows, i32(full, device), i32(ctx, device), i32(cu, device),
                          i32(A.prompt_tiles(cu, ctx, a.H, a.G, n_rows), device))
        close(got, torch.cat([w[lo:hi] for w, (lo, hi) in zip(want, cuts)]), limit)
    for ctx in ([300, 131], [1, 2], [32, 33], [64, 65], [41, 40], [97, 128], [34, 100]):
        q = torch.stack([s[1][c - 1] for s, c in zip(seqs, ctx)])
        for P in (1, 3, 7):
            got = A.attention(a, packed_q(a, q, dtype, device), rows, i32(full, device), i32(ctx, device), P=P)
            close(got, torch.stack([w[c - 1] for w, c in zip(want, ctx)]), limit)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("pool", [0, 8])
def test_single_keys_at_edges(device, dtype, pool):
    """One key (or one block's mean) scores far above all others, its value marked: rows just inside its sight give the
    value back, rows just outside do not -- at page borders, window edges, the kept tokens' end."""
    size, keep, T = 48, 0 if pool else 6, 200
    a = heads_of(4, 2, 64, 64, True, 0, 0, A.Mask(size, keep, pool), device=device, sink=False)
    table = [6, 1, 5, 0, 3, 2, 4]
    for p in (0, 5, 6, 31, 32, 63, 64, 100):
        rows = PagedHeads(7, 2, a.D, pool, A.pool_entries(pool) if pool else 0, device, dtype)
        q, k, v = torch.ones(T, 4, 64), 0.02 * rnd(T, 2, 64, seed=p), torch.zeros(T, 2, 64)
        k[p], v[p] = 8.0, 100.0
        fill(a, rows, k, v, table, device)
        want = want_attn(a, q, k, v, dtype)
        first = (p // pool + 1) * pool - 1 + size if pool else T
        for t in sorted({p, p + 1, p + size - 1, p + size, first - 1, first, T - 1}):
            if not p <= t < T:
                continue
            seen = t - p < size or p < keep or t >= first
            assert bool(want[t].max() > 5) == seen, (p, t)
            got = A.attention(a, packed_q(a, q[t:t + 1], dtype, device), rows, i32([table], device), i32([t + 1], device))
            close(got, want[t:t + 1], 1.5e-2 if dtype == torch.bfloat16 else 3e-5)
            lo = max(0, t - 3)
            got = A.attention(a, packed_q(a, q[lo:t + 1], dtype, device), rows, i32([table], device), i32([t + 1], device),
                              i32([0, t + 1 - lo], device), i32(A.prompt_tiles([0, t + 1 - lo], [t + 1], 4, 2, A.prompt_rows(dtype, a.D)), device))
            close(got, want[lo:t + 1], 1.5e-2 if dtype == torch.bfloat16 else 3e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_sink_counts_once(device, dtype):
    """Equal scores of zero: the sink's weight against the visible keys alone, over both ranges and all slices."""
    for mask, seen in ((A.Mask(10, keep=2), 12), (A.Mask(10, pool=4), 10 + 91 // 4), (A.Mask(0), 100)):
        a = heads_of(2, 1, 32, 32, True, 0, 0, mask, device=device)
        a.sink = torch.tensor([1.5, -0.5], device=device)
        rows = PagedHeads(4, 1, a.D, mask.pool, A.pool_entries(mask.pool) if mask.pool else 0, device, dtype)
        fill(a, rows, torch.zeros(100, 1, 32), torch.ones(100, 1, 32), [2, 0, 3, 1], device)
        for P in (1, 4):
            got = A.attention(a, torch.zeros(1, 2, 32, dtype=dtype, device=device), rows, i32([[2, 0, 3, 1]], device), i32([100], device), P=P)
            close(got.view(2, 32)[:, 0], torch.tensor([seen / (seen + math.exp(s)) for s in (1.5, -0.5)]), 1e-5 if dtype == torch.float32 else 4e-3)


def test_prompt_rows_match_the_kernel():
    from copilot_for_consensus_amd.ops import _native
    if not _native.kernels_available():
        pytest.skip("kernels not built")
    for d in range(32, 1025, 32):
        assert _native.kernels().cfc_gqa_prompt_rows(d) == A.prompt_rows(torch.bfloat16, d)


# ------------------------------------------------------------------ routing and experts
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,top", [(10, 4), (3, 3), (70, 5), (300, 9), (1, 1)])
def test_softmax_routing(device, E, top):
    T, W = 33, 24
    h, p = rnd(T, W), {"router": rnd(E, W, seed=1), "correction": 0.2 * rnd(E, seed=2) - 0.1}
    ids, weights = oracle.route(h, p, top)
    r = M.Router(E, top, 1, 1, 1.0, p["correction"].to(device), softmax=True, renorm=False)
    z = torch.cat([torch.zeros(T, 4), h @ p["router"].T], 1)
    gi, gw = M.route(Cols(slabs(z, 3).to(device), 4, E), r)
    for t in range(T):
        got = dict(zip(gi[t].tolist(), gw[t].tolist()))
        want = dict(zip(ids[t], map(float, weights[t])))
        assert got.keys() == want.keys() and all(abs(got[e] - want[e]) < 1e-5 for e in got), t


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,F,W,T,top", [(6, 24, 64, 40, 3), (6, 72, 128, 2, 3), (5, 64, 192, 300, 2), (3, 20, 65, 9, 2), (4, 128, 64, 900, 2)])
def test_experts_with_identity_choices(device, dtype, E, F, W, T, top):
    """Clamped experts, choices past the last one on the rows' own input; a batch that chooses nothing else; through the
    sort, the grouped products and the branch."""
    x = rnd(T, W).to(dtype)
    p = {f"e{e}.{k}": rnd(*((F, W) if k != "down" else (W, F)), seed=3 * e + j, scale=1.5 / W ** 0.5).to(dtype)
         for e in range(E) for j, k in enumerate(("gate", "up", "down"))}
    w = M.ExpertWeights(*(torch.stack([p[f"e{e}.{k}"] for e in range(E)]).to(device) for k in ("gate", "up", "down")))
    g = torch.Generator().manual_seed(3)
    for ids in (torch.stack([torch.randperm(E + 2, generator=g)[:top] for _ in range(T)]), torch.full((T, top), E)):
        wt = torch.rand(T, top, generator=g)
        q = {k: v.float() for k, v in p.items()}
        want = torch.stack([sum(wt[t, c] * (x[t].float() if ids[t, c] >= E else oracle.expert(x[t].float(), q, f"e{int(ids[t, c])}", 0.9))
                                for c in range(top)) for t in range(T)])
        di = i32(ids, device)
        rows, pos = M.experts(x.to(device), w, di, M.Glu(0.9, 1.702, 1.0))
        stream = torch.zeros(T, W, device=device)
        br = N.Branch(torch.ones(1, device=device), 1e-3, routed=(rows, pos, wt.to(device), di, E, x.to(device)))
        N.branch_norm(stream, br, None, 1e-3, None)
        close(stream, oracle.rms(want, 1e-3), 3e-5 if dtype == torch.float32 else 3e-2)


@pytest.mark.parametrize("device", [pytest.param("cuda", marks=pytest.mark.gpu)])
@pytest.mark.parametrize("T,top,E,tile", [(5, 2, 4, 64), (300, 3, 7, 64), (700, 4, 5, 128)])
def test_sorting_skips_choices_without_matrices(device, T, top, E, tile):
    ids = torch.randint(0, E + 3, (T, top), generator=torch.Generator().manual_seed(T), dtype=torch.int32)
    rows, pos, te = M.sort_rows(ids.to(device), E, tile)
    wr, wp, wt = moe_rows(ids, E, tile)
    assert torch.equal(te.cpu(), torch.from_numpy(wt)) and torch.equal(pos.cpu(), torch.from_numpy(wp))
    live = torch.from_numpy(np.repeat(wt >= 0, tile))
    assert torch.equal(rows.cpu()[live], torch.from_numpy(wr)[live])
