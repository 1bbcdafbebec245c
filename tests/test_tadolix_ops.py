"""Each mechanism of the Tadolix decoder alone, against the plain implementation."""
import math

import numpy as np
import pytest
import torch

import tadolix_oracle as oracle
from copilot_for_consensus_amd.models.projection import Projection
from copilot_for_consensus_amd.models.tadolix import GELU
from copilot_for_consensus_amd.ops import gqa as A
from copilot_for_consensus_amd.ops import gru as R
from copilot_for_consensus_amd.ops import hyper as X
from copilot_for_consensus_amd.ops import rglru as L
from copilot_for_consensus_amd.ops import stream as S
from copilot_for_consensus_amd.ops.cols import Cols
from copilot_for_consensus_amd.ops.reference import interleave_gate_up
from copilot_for_consensus_amd.runtime.kv_cache import PagedHeads

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(autouse=True)
def one_thread():
    """The CPU cases are many small operations: threads only get in each other's way."""
    n = torch.get_num_threads()
    torch.set_num_threads(1)
    yield
    torch.set_num_threads(n)


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


# ------------------------------------------------------------------ embedding
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [64, 65, 300])
def test_embedding_with_sinusoids(device, dtype, W):
    table, T = rnd(50, W).to(dtype), 40
    ids = torch.randint(0, 50, (T,), generator=torch.Generator().manual_seed(1), dtype=torch.int32)
    want = oracle.embedding(table.float(), ids.long(), 7.5)
    got = S.embed_f32(table.to(device), ids.to(device), torch.empty(T, W, device=device), 7.5, i32(range(T), device),
                      S.sinusoid_turns(W, 10000.0, device))
    close(got, want, 1e-6)


# ------------------------------------------------------------------ hyper-connections
def connection(n, device, seed):
    c = [rnd(n, seed=seed), rnd(n, n, seed=seed + 1), rnd(n, seed=seed + 2)]
    return c, X.Connection(*(t.to(device) for t in c))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,W,T,split", [(1, 104, 5, 1), (2, 65, 3, 3), (3, 300, 2, 2), (4, 1500, 4, 9), (4, 4096, 3, 4), (4, 5000, 2, 2), (7, 260, 3, 1),
                                         (16, 64, 2, 2), (16, 33, 2, 1)])
def test_streams_over_several_sublayers(device, dtype, n, W, T, split):
    """From one row for all streams on; every kind of reading in turn, the pending result added once each time."""
    e, eps = 2 * rnd(T, W), 1e-2
    xs, got = [e] * n, X.Streams(e.to(device), n)
    h = torch.empty(T, W, dtype=dtype, device=device)
    for q in range(4):
        (inp, mix, out), c = connection(n, device, 10 * q)
        w, y = rnd(W, seed=5 + q), rnd(T, W, seed=50 + q)
        row = oracle.read_streams(xs, inp)
        if q % 2:
            X.norm(got, c.inp, (1.0 + w).to(device), eps, h)
            close(h, oracle.norm(row, w, eps), tol(dtype))
        else:
            u, rstd = torch.empty(T, W, device=device), torch.empty(T, device=device)
            X.stats(got, c.inp, eps, u, rstd)
            close(u, row, 2e-5)
            close(u.cpu() * rstd.cpu()[:, None], oracle.rms(row, eps), 2e-5)
        assert got.done is None
        got.done = (slabs(y, split, seed=q).to(device), c)
        xs = oracle.write_streams(xs, y, mix, out)
    want, w = oracle.norm(sum(xs), rnd(W, seed=5), eps), (1.0 + rnd(W, seed=5)).to(device)
    if device == "cuda":                                     # not stored: may be read again
        close(X.last_norm(got, w, eps, dtype, i32([T - 1, 0], device)), want[[T - 1, 0]], tol(dtype))
    close(X.last_norm(got, w, eps, dtype), want, tol(dtype))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps,W", [(1, 64), (2, 65), (3, 104), (4, 260), (7, 96), (4, 4200), (35, 64)])
def test_input_convolution_in_portions_and_decoded(device, dtype, taps, W):
    """Portions of every kind, two sequences at once, then decoded rows, in a used slot; other slots untouched."""
    T, eps = 90, 1e-2
    rows, w, k = [rnd(T, W, seed=s) for s in (1, 2)], rnd(W, seed=3), rnd(W, taps, seed=4)
    want = [oracle.input_conv(oracle.norm(x, w, eps), k) for x in rows]
    tail = rnd(5, taps - 1, W, seed=6).to(device) if taps > 1 else None
    before = tail.clone() if taps > 1 else None
    slots, one = [3, 1], torch.ones(1, device=device)
    conv, wd = k.t().contiguous().to(device), (1.0 + w).to(device)
    at = [0, 0]
    for cuts in ([37, 2], [2, 33], [1, 1], [3, 34], [27, 1], [1, 1], [1, 1], [1, 1], [1, 1]):
        x = torch.cat([r[a:a + n] for r, a, n in zip(rows, at, cuts)])
        por, lo = [], 0
        for s, n in enumerate(cuts):
            por.append((lo, n, at[s], s))
            lo += n
        h = torch.empty(lo, W, dtype=dtype, device=device)
        xs, t = X.Streams(x.to(device), 1), S.Tail(tail, i32(slots, device))
        if max(cuts) > 1:
            u, rstd = torch.empty(lo, W, device=device), torch.empty(lo, device=device)
            X.stats(xs, one, eps, u, rstd)
            S.input_conv(u, rstd, wd, [conv], i32(S.conv_tiles(por, max(32, taps - 1)), device), t, [h])
        else:
            X.conv_decode(xs, one, wd, eps, conv, i32(at, device), t, h)
        close(h, torch.cat([v[a:a + n] for v, a, n in zip(want, at, cuts)]), tol(dtype))
        at = [a + n for a, n in zip(at, cuts)]
    if taps > 1:
        assert torch.equal(tail[[0, 2, 4]], before[[0, 2, 4]])


def test_tiles_of_a_convolution_with_slots():
    """Cut from the portion's start on, so that only its first tile reads what lies before it."""
    t = S.conv_tiles([(0, 70, 31, 0), (70, 1, 5, 1)], 32)
    assert t[0].tolist() == [[0, 32, 31, 0], [32, 32, 63, 0], [64, 6, 95, 0], [70, 1, 5, 1]]
    assert t[1, :, :2].tolist() == [[0, 70], [32, 70], [64, 70], [0, 1]]


# ------------------------------------------------------------------ feed-forward
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,F,split,inter", [(3, 33, 2, False), (5, 256, 3, True), (2, 1032, 1, True)])
def test_gelu_gate(device, dtype, T, F, split, inter):
    g, u = rnd(T, F, scale=3.0), rnd(T, F, seed=1)
    g[0, :4] = torch.tensor([-40.0, 40.0, 0.0, -1e4])
    gu = torch.cat([g, u], 1)
    if inter:
        gu = interleave_gate_up(gu.T.contiguous()).T.contiguous()
    got = S.clamped_glu(slabs(gu, split).to(device), torch.empty(T, F, dtype=dtype, device=device), **GELU, interleaved=inter)
    close(got, oracle.gelu_tanh(g) * u, 1e-5 if dtype == torch.float32 else 1.2e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("M,F,K", [(300, 12352, 128), (2, 128, 64), (513, 12800, 192), (100, 128, 320), (64, 16384, 128)])
def test_gelu_gate_of_a_product(M, F, K):
    """Every kernel a gated product takes, among them the prompt and decode products' epilogues."""
    x, gu = rnd(M, K).to(torch.bfloat16), rnd(2 * F, K, seed=1, scale=2 * K ** -0.5).to(torch.bfloat16)
    y = x.float() @ gu.float().T
    got = Projection(interleave_gate_up(gu.cuda()), swiglu=True).glu(x.cuda(), torch.empty(M, F, dtype=torch.bfloat16, device="cuda"), **GELU)
    close(got, oracle.gelu_tanh(y[:, :F]) * y[:, F:], 8e-3)


# ------------------------------------------------------------------ distance bias
def test_distance_table_rows():
    """Against logarithms away from a step's edge, and exactly on it; odd tables, tables of two rows, fractional ends."""
    for rows, far in ((32, 240), (32, 128), (7, 17), (10, 100), (2, 5), (16, 256), (3, 2), (24, 60.5), (1, 9), (64, 33)):
        starts = A.distance_starts(rows, far)
        assert len(starts) == rows and starts == sorted(starts) and starts[0] == 0
        for n in range(int(1.2 * far) + 3):
            b, half = oracle.bucket(n, rows, far) if rows > 1 else 0, rows // 2
            assert b == max(i for i, s in enumerate(starts) if s <= n), (rows, far, n)
            if n >= half > 0 and rows > 2:
                f = math.log(n / half) / math.log(far / half) * (rows - half)
                assert min(rows - 1, half + math.floor(f)) == b or abs(f - round(f)) < 1e-9
    with pytest.raises(ValueError):
        A.distance_starts(32, 16)
    rel = rnd(10, 3)
    for limit in (0, 200, 30, 1):
        t = A.distance_bias(rel, 100, limit)
        assert t.shape[0] == 3 and (not limit or t.shape[1] <= limit)
        for n in range(limit or 300):
            assert torch.equal(t[:, min(n, t.shape[1] - 1)], rel[oracle.bucket(n, 10, 100)])


# ------------------------------------------------------------------ attention
ATTN = [  # H, G, dim, vdim, scale, cap, rows of the table, its far end, chunk
    (4, 2, 64, 64, 0.2, 50.0, 32, 120, 100), (6, 2, 48, 40, 0.25, 45.0, 16, 50, 56), (3, 1, 18, 14, 1.0, 5.0, 7, 17, 17),
    (2, 2, 36, 9, 0.4, 0.0, 10, 40, 70), (20, 1, 128, 128, 0.09, 50.0, 32, 200, 290), (40, 1, 32, 32, 0.5, 3.0, 4, 6, 1),
    (2, 1, 140, 160, 0.09, 40.0, 32, 500, 0), (4, 2, 64, 64, 0.2, 60.0, 12, 70, 128), (2, 1, 192, 180, 0.1, 8.0, 2, 5, 65), (1, 1, 256, 256, 0.06, 50.0, 20, 90, 150),
    (2, 2, 300, 33, 0.06, 30.0, 32, 100, 45), (24, 1, 64, 62, 0.2, 60.0, 40, 400, 0), (4, 4, 96, 96, 0.1, 30.0, 1, 9, 33)]


def attn_case(case, device):
    H, G, dim, vdim, scale, cap, rows, far, chunk = case
    rel = rnd(rows, H, seed=3, scale=1.5).to(torch.bfloat16).float()
    one = torch.ones(dim, device=device)
    return rel, A.Heads(H, G, dim, vdim, scale, A.Mask(chunk, chunked=chunk > 0), 1e-3, one, one, True, None, softcap=cap,
                        bias=A.distance_bias(rel, far, chunk).to(device), unit=True)


def unit(x):
    return oracle.rms(x, 1e-3)


def fill(a, rows, k, v, table, device):
    for i in range(k.shape[0]):
        rows.k[table[i // 32], :, i % 32, :a.dim] = k[i].to(rows.k.dtype).to(device)
        rows.v[table[i // 32], :, i % 32, :a.vdim] = v[i].to(rows.v.dtype).to(device)


def packed_q(a, q, dtype, device):
    out = torch.zeros(q.shape[0], a.H, a.D, dtype=dtype, device=device)
    out[..., :a.dim] = (q * a.q_scale).to(dtype).to(device)
    return out


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", ATTN)
def test_attention_in_portions_and_decoded(device, dtype, case):
    """Two sequences at once: a whole prompt, portions at page, tile and chunk edges, and single tokens in one and in
    several key slices; gated or not, into rows of another's width; garbage pages in the pool do not matter."""
    H, G, dim, vdim, scale, cap, _, far, chunk = case
    rel, a = attn_case(case, device)
    assert a.capped == (0 if not cap else 3 if dim * scale <= 0.24 * cap else 2 if dim * scale <= 0.34 * cap else 1)
    lens, tables = [300, 131], [[3, 9, 1, 14, 7, 5, 11, 0, 8, 2], [13, 4, 6, 12, 10]]
    rows = PagedHeads(16, G, a.D, 0, 0, device, dtype)
    for t, w in ((rows.k, dim), (rows.v, vdim)):
        t.normal_(0.0, 1.0)                                 # what other sequences left
        t[..., w:] = 0.0
    qs, want = [], []
    for s, (n, table) in enumerate(zip(lens, tables)):
        q, k, v = unit(rnd(n, H, dim, seed=21 + s)), unit(rnd(n, G, dim, seed=31 + s)), rnd(n, G, vdim, seed=41 + s)
        fill(a, rows, k, v, table, device)
        # what the kernels read: rounded queries and rows
        k, v = k.to(dtype).float(), v.to(dtype).float()
        qr = (q * a.q_scale).to(dtype).float() / a.q_scale
        want.append(oracle.attend(qr, k, v, scale, cap, rel, far, chunk))
        qs.append(q)
    gates = [rnd(n, H * vdim, seed=61 + s).to(dtype).float() for s, n in enumerate(lens)]
    full = [t + [0] * (10 - len(t)) for t in tables]
    limit = 3e-5 if dtype == torch.float32 else 1.5e-2

    def both(ranges):
        return (torch.cat([x[s][lo:hi] for s, (lo, hi) in enumerate(ranges)]) for x in (qs, want, gates))
    for i, cuts in enumerate(([(0, 300), (0, 131)], [(63, 66), (0, 2)], [(64, 129), (31, 33)], [(299, 300), (40, 131)], [(33, 290), (128, 131)])):
        q, w, g = both(cuts)
        cu, ctx = np.cumsum([0] + [hi - lo for lo, hi in cuts]).tolist(), [hi for _, hi in cuts]
        buf = torch.full((cu[-1], H * vdim + 12), 7.0, dtype=dtype, device=device)
        args = dict(cu_q=i32(cu, device), tiles=i32(A.prompt_tiles(cu, ctx, H, G, A.prompt_rows(dtype, a.D)), device))
        if i % 2 == 0:
            args |= dict(gate=Cols(g.to(device, dtype)), factor=0.6, out=buf[:, 8:8 + H * vdim])
            w = w * 0.6 * torch.sigmoid(g)
        got = A.attention(a, packed_q(a, q, dtype, device), rows, i32(full, device), i32(ctx, device), **args)
        close(got, w, limit)
        assert (buf[:, :8] == 7).all() and (buf[:, 8 + H * vdim:] == 7).all()
    for i, ctx in enumerate(([300, 131], [1, 2], [32, 33], [64, 65], [97, 128], [34, 100], [290, 17])):
        q, w, g = both([(c - 1, c) for c in ctx])
        for P in (1, 3, 7):
            args = {}
            if i % 2 == 0:
                args = dict(gate=Cols(slabs(torch.cat([torch.zeros(2, 4), g], 1), 3).to(device), 4), factor=-1.5)
            got = A.attention(a, packed_q(a, q, dtype, device), rows, i32(full, device), i32(ctx, device), P=P, **args)
            close(got, w * -1.5 * torch.sigmoid(g) if args else w, limit)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_single_keys_at_chunk_edges(device, dtype):
    """One key scores far above all others, its value marked: rows of its chunk give the value back, rows of the next do
    not -- at page borders, chunk edges, and beside keys at the table's last distances."""
    size, T, rel = 48, 200, torch.zeros(8, 4)
    rel[7] = 1.0
    a = A.Heads(4, 2, 64, 64, 0.3, A.Mask(size, chunked=True), 1e-3, None, None, True, None, softcap=40.0, bias=A.distance_bias(rel, 30, size).to(device))
    assert a.capped == 1
    table = [6, 1, 5, 0, 3, 2, 4]
    for p in (0, 31, 32, 47, 48, 63, 64, 95, 96, 100):
        rows = PagedHeads(7, 2, a.D, 0, 0, device, dtype)
        q, k, v = torch.ones(T, 4, 64), 0.02 * rnd(T, 2, 64, seed=p), torch.zeros(T, 2, 64)
        k[p], v[p] = 2.0, 100.0
        fill(a, rows, k, v, table, device)
        qr = (q * a.q_scale).to(dtype).float() / a.q_scale
        want = oracle.attend(qr, k.to(dtype).float(), v, 0.3, 40.0, rel, 30, size)
        edge = (p // size + 1) * size
        for t in sorted({p, p + 1, edge - 1, edge, edge + 1, T - 1}):
            assert bool(want[t].max() > 5) == (t < edge), (p, t)
            got = A.attention(a, packed_q(a, q[t:t + 1], dtype, device), rows, i32([table], device), i32([t + 1], device))
            close(got, want[t:t + 1], 1.5e-2 if dtype == torch.bfloat16 else 3e-5)
            lo = max(0, t - 3)
            got = A.attention(a, packed_q(a, q[lo:t + 1], dtype, device), rows, i32([table], device), i32([t + 1], device),
                              i32([0, t + 1 - lo], device), i32(A.prompt_tiles([0, t + 1 - lo], [t + 1], 4, 2, A.prompt_rows(dtype, a.D)), device))
            close(got, want[lo:t + 1], 1.5e-2 if dtype == torch.bfloat16 else 3e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_kept_tokens_beside_a_chunk(device, dtype):
    """The first tokens stay in sight of later chunks (a mask the kernels also take), with their distances' bias."""
    rel, size, keep, T = rnd(12, 2, seed=5), 40, 5, 170
    a = A.Heads(2, 1, 32, 32, 0.3, A.Mask(size, keep, chunked=True), 1e-3, None, None, True, None, bias=A.distance_bias(rel, 60, 0).to(device))
    q, k, v = rnd(T, 2, 32, seed=1), rnd(T, 1, 32, seed=2).to(dtype).float(), rnd(T, 1, 32, seed=3).to(dtype).float()
    rows, table = PagedHeads(6, 1, a.D, 0, 0, device, dtype), [2, 5, 0, 3, 1, 4]
    fill(a, rows, k, v, table, device)
    qr, j = (q * a.q_scale).to(dtype).float() / a.q_scale, torch.arange(T)
    see = oracle.chunk_mask(T, size) | ((j[None] < keep) & (j[None] <= j[:, None]))
    bias = rel[torch.tensor([oracle.bucket(n, 12, 60) for n in range(T)])][(j[:, None] - j[None]).clamp(min=0)]
    want = torch.cat([torch.softmax((qr[:, h] @ k[:, 0].T * 0.3 + bias[..., h]).masked_fill(~see, -math.inf), 1) @ v[:, 0] for h in range(2)], 1)
    limit = 3e-5 if dtype == torch.float32 else 1.5e-2
    got = A.attention(a, packed_q(a, q, dtype, device), rows, i32([table], device), i32([T], device), i32([0, T], device),
                      i32(A.prompt_tiles([0, T], [T], 2, 1, A.prompt_rows(dtype, a.D)), device))
    close(got, want, limit)
    for t in (0, 3, 39, 40, 44, 45, 120, 169):
        for P in (1, 3):
            got = A.attention(a, packed_q(a, q[t:t + 1], dtype, device), rows, i32([table], device), i32([t + 1], device), P=P)
            close(got, want[t:t + 1], limit)


# ------------------------------------------------------------------ gated recurrence into wider rows
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,at", [(33, 5), (96, 64), (1024, 128)])
def test_gated_recurrence_scaled_into_wider_rows(device, dtype, W, at):
    T = 150
    z, u, g = (rnd(T, W, seed=s, scale=2.0).to(dtype).float() for s in (1, 2, 3))
    bz, bx = rnd(W, seed=4) - 2.0, rnd(W, seed=5)
    want = -0.3 * oracle.min_gru((z + bz).double(), (u + bx).double()).float() * g * torch.sigmoid(g)
    p, zug = R.Gru(bz.to(device), bx.to(device)), torch.cat([z, u, g], 1).to(device, dtype)
    state, buf = rnd(3, W, seed=6).to(device), torch.full((T, at + W + 4), 7.0, dtype=dtype, device=device)
    n = T - 3
    ch, cu = R.chunk_plan([0, n])
    R.prefill(p, *(Cols(zug[:n], k * W, W) for k in range(3)), i32([2], device), i32([0, n], device), i32([n], device), i32(ch, device),
              i32(cu, device), state, buf[:n, at:at + W], -0.3)
    for t in range(n, T):
        c = torch.cat([z[t:t + 1], u[t:t + 1], g[t:t + 1]], 1)
        R.step(p, *(Cols(slabs(c, 2).to(device), k * W, W) for k in range(3)), i32([2], device), i32([t + 1], device), state, buf[t:t + 1, at:at + W],
               -0.3)
    close(buf[:, at:at + W], want, tol(dtype))
    assert (buf[:, :at] == 7).all() and (buf[:, at + W:] == 7).all()


# ------------------------------------------------------------------ real-gated linear recurrence
def lru_case(width, blocks, taps, dtype, device, lam=None):
    b = width // blocks
    p = {"x.b": rnd(width, seed=1), "conv": rnd(width, taps, seed=2, scale=0.7), "conv.b": 0.3 * rnd(width, seed=3),
         "ra": rnd(blocks, b, b, seed=4, scale=1.5 * b ** -0.5).to(dtype).float(), "ra.b": rnd(blocks, b, seed=5),
         "ri": rnd(blocks, b, b, seed=6, scale=1.5 * b ** -0.5).to(dtype).float(), "ri.b": rnd(blocks, b, seed=7),
         "lam": 2.0 * rnd(width, seed=8) - 4.0 if lam is None else torch.full((width,), lam), "y.b": rnd(width, seed=9)}
    rate = -8.0 * torch.nn.functional.softplus(p["lam"].double()).float()
    d = lambda t: t.to(device).contiguous()
    return p, L.RgLru(d(p["x.b"]), d(p["conv"].T), d(p["conv.b"]), d(p["ra"].to(dtype)), d(p["ra.b"].view(-1)), d(p["ri"].to(dtype)),
                      d(p["ri.b"].view(-1)), d(rate), d(p["y.b"]))


def want_lru(p, x, y, dtype):
    u = (oracle.short_conv(x + p["x.b"], p["conv"]) + p["conv.b"]).to(dtype).double()      # the activations' rounding
    q = {k: v.double() for k, v in p.items()}
    S = oracle.rglru(u, oracle.block_gate(u, q["ra"], q["ra.b"]), oracle.block_gate(u, q["ri"], q["ri.b"]), q["lam"])
    return (S * oracle.gelu_tanh((y + p["y.b"]).double())).float()


LRU = [(64, 2, 4, None), (60, 3, 3, None), (35, 5, 6, None), (7, 1, 1, None), (160, 2, 3, None), (192, 2, 2, -9.0), (256, 1, 4, 1.0), (1024, 4, 4, None),
       (300, 1, 2, None), (520, 1, 3, None), (1100, 1, 2, None), (96, 96, 4, None), (264, 3, 4, -12.0)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", LRU)
def test_linear_recurrence_in_portions_and_decoded(device, dtype, case):
    """Whole, in portions down to one token that carry state and convolution, then token by token; a batch of several
    sequences; slots that hold others' values, and others' slots untouched."""
    W, blocks, taps, lam = case
    T = 290
    p, r = lru_case(W, blocks, taps, dtype, device, lam)
    x, y = (rnd(T, W, seed=s).to(dtype).float() for s in (11, 12))
    want, yx = want_lru(p, x, y, dtype), torch.cat([y, x], 1).to(device, dtype)
    limit = 5e-5 if dtype == torch.float32 else 2e-2

    def portions(ranges, slots, tail, state, whole=False):
        idx = torch.cat([torch.arange(lo, hi) for lo, hi in ranges])
        cu = np.cumsum([0] + [hi - lo for lo, hi in ranges]).tolist()
        por = [(cu[s], hi - lo, lo, s) for s, (lo, hi) in enumerate(ranges)]
        seg, seg_cu = (None, None) if whole else (i32(t, device) for t in R.chunk_plan(cu, L.SEGMENT))
        rows = yx[idx.to(device)].contiguous()
        out = L.prefill(r, Cols(rows, W, W), Cols(rows, 0, W), i32(slots, device), i32(cu, device), i32([hi for _, hi in ranges], device),
                        i32(S.conv_tiles(por, 32), device), seg, seg_cu, tail, state,
                        torch.empty(cu[-1], W, dtype=dtype, device=device))
        close(out, want[idx], limit)

    for cuts in ([290], [128, 1, 2, 127, 32], [1, 1, 130, 3]):
        tail, state = rnd(4, r.ring, W, seed=6).to(device), rnd(4, W, seed=6).to(device)
        before, at = (tail.clone(), state.clone()), 0
        for n in cuts:
            portions([(at, at + n)], [2], tail, state)
            at += n
        # decoded from where the portions ended, beside a sequence that starts
        for t in range(at, min(at + 12, T)):
            both, first = [t, t - at], t == at
            rows = torch.cat([y[both], x[both]], 1)
            c = slabs(rows, 3, seed=t).to(device)
            out = L.step(r, Cols(c, W, W), Cols(c, 0, W), i32([2, 0], device), i32(both, device), i32([b + 1 for b in both], device), tail, state,
                         torch.empty(2, W, dtype=dtype, device=device))
            close(out, want[both], limit)
        assert torch.equal(state[[1, 3]], before[1][[1, 3]]) and torch.equal(tail[[1, 3]], before[0][[1, 3]])
    tail, state = rnd(4, r.ring, W, seed=7).to(device), rnd(4, W, seed=8).to(device)
    for whole in (False, True):
        portions([(0, 150), (0, 1), (0, 257)], [3, 0, 2], tail, state, whole)
        portions([(150, 152), (1, 34), (257, 290)], [3, 0, 2], tail, state, whole)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", [(35, 5, 3), (192, 2, 4), (800, 8, 5), (260, 1, 2)])
def test_linear_recurrence_of_many_decoded_rows(device, dtype, case):
    """More rows than a tile, each at another position of its own sequence, slots in any order."""
    W, blocks, taps = case
    B = 37
    p, r = lru_case(W, blocks, taps, dtype, device)
    seqs = [(rnd(9, W, seed=2 * b).to(dtype).float(), rnd(9, W, seed=2 * b + 1).to(dtype).float()) for b in range(B)]
    want = [want_lru(p, x, y, dtype) for x, y in seqs]
    slots = torch.randperm(B + 2, generator=torch.Generator().manual_seed(1))[:B].tolist()
    tail, state = rnd(B + 2, r.ring, W, seed=6).to(device), rnd(B + 2, W, seed=7).to(device)
    for t in range(9):
        rows = [b for b in range(B) if b % 9 <= t]            # sequence b starts at step b % 9
        at = [t - b % 9 for b in rows]
        c = slabs(torch.stack([torch.cat([seqs[b][1][i], seqs[b][0][i]]) for b, i in zip(rows, at)]), 5, seed=t).to(device)
        out = L.step(r, Cols(c, W, W), Cols(c, 0, W), i32([slots[b] for b in rows], device), i32(at, device), i32([i + 1 for i in at], device),
                     tail, state, torch.empty(len(rows), W, dtype=dtype, device=device))
        close(out, torch.stack([want[b][i] for b, i in zip(rows, at)]), 5e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("device", DEVICES)
def test_decays_near_one_keep_their_digits(device):
    """The slowest decays: 1 - a^2 far below a's rounding, over a long portion."""
    T, W = 512, 64
    for dtype in DTYPES:
        p, r = lru_case(W, 2, 1, dtype, device, -14.0)
        p["ra.b"] -= 6.0
        r.ra_b -= 6.0
        x, y = torch.ones(T, W), torch.ones(T, W)
        want, yx = want_lru(p, x, y, dtype), torch.ones(T, 2 * W, dtype=dtype, device=device)
        seg, cu = R.chunk_plan([0, T], L.SEGMENT)
        out = L.prefill(r, Cols(yx, W, W), Cols(yx, 0, W), i32([0], device), i32([0, T], device), i32([T], device),
                        i32(S.conv_tiles([(0, T, 0, 0)], 32), device), i32(seg, device), i32(cu, device), torch.zeros(1, 1, W, device=device),
                        torch.zeros(1, W, device=device), torch.empty(T, W, dtype=dtype, device=device))
        close(out / want.abs().amax().to(device), want / want.abs().amax(), 1e-4 if dtype == torch.float32 else 2e-2)


def test_portions_as_segments():
    assert L.whole_portions([0, 1, 129], 64) and not L.whole_portions([0, 2800], 4096)
    assert L.whole_portions(list(range(0, 6 * 2800 + 1, 2800)), 4096) and not L.whole_portions([0, 5000] + list(range(5001, 5016)), 4096)


def test_segments_match_the_kernels():
    from copilot_for_consensus_amd.ops import _native
    if not _native.kernels_available():
        pytest.skip("kernels not built")
    assert _native.kernels().cfc_rglru_segment() == L.SEGMENT and _native.kernels().cfc_rglru_max_block() == L.MAX_BLOCK
