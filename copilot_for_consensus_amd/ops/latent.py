"""Latent attention ops (csrc/kernels/latent.hip): the norms of both latents with the cache write, the
per-head products around the attention, and attention over the paged latents.

GPU tensors go to the native library (which must be built), CPU tensors to the fp32 reference.
"""
from __future__ import annotations

import dataclasses
import math

import numpy as np
import torch

from . import reference as ref
from ._native import check, kernels
from .cols import Cols
from .kernels import _p, _req, _stream, _workspace
from .stream import _act

MFMA_MAX_RANK = 512       # latent ranks the MFMA attention kernel is built for
MFMA_MAX_KEY = 576        # and key columns (the latent and what follows it in the row)
ANY_ROWS = 4              # rows per tile of the general kernel


def padded_rank(rank: int) -> int:
    """Latent row stride: the rank rounded up to one MFMA step (32); the pad columns stay zero."""
    return 32 * math.ceil(rank / 32)


class HeadWeight:
    """Per-head matrices [H, N, K] zero-padded to [H, 64 x, 32 y] for :func:`head_linear`."""

    __slots__ = ("data", "H", "N", "K")

    def __init__(self, w: torch.Tensor, n_out: int | None = None, k_in: int | None = None):
        H, N, K = w.shape
        self.H, self.N, self.K = H, n_out or N, k_in or K
        self.data = torch.zeros(H, 64 * math.ceil(self.N / 64), 32 * math.ceil(self.K / 32), dtype=w.dtype, device=w.device)
        self.data[:, :N, :K] = w

    def nbytes(self) -> int:
        return self.data.numel() * self.data.element_size()


def head_linear(x: torch.Tensor, w: HeadWeight, out: torch.Tensor, gate: torch.Tensor | None = None) -> torch.Tensor:
    """out[t, h, :N] = w[h] x[t, h, :K], times sigmoid(gate[t, h N + n]) when given ([T, H N], row-strided).
    x [T, H, >= K], out [T, H, >= N]: any row / head strides, last dim dense."""
    T, H = x.shape[0], x.shape[1]
    if H != w.H or out.shape[:2] != (T, H) or x.shape[2] < w.K or out.shape[2] < w.N:
        raise ValueError(f"head_linear: x {tuple(x.shape)} w {w.H} x {w.N} x {w.K} out {tuple(out.shape)}")
    if not x.is_cuda:
        y = torch.matmul(x[:, :, :w.K].float().transpose(0, 1), w.data[:, :w.N, :w.K].float().transpose(1, 2))
        y = y.transpose(0, 1)
        if gate is not None:
            y = y * torch.sigmoid(gate.float().view(T, H, w.N))
        out[:, :, :w.N] = y.to(out.dtype)
        return out
    if x.stride(2) != 1 or out.stride(2) != 1 or x.dtype != out.dtype or x.dtype != w.data.dtype:
        raise ValueError("head_linear: dense last dimensions and one dtype needed")
    if gate is not None and (gate.shape != (T, H * w.N) or gate.stride(1) != 1 or gate.dtype != x.dtype):
        raise ValueError(f"head_linear: gate {tuple(gate.shape)} {gate.dtype}")
    check(kernels().cfc_head_linear(_act(x.dtype), x.data_ptr(), x.stride(0), x.stride(1), w.data.data_ptr(),
                                    w.data.shape[1], w.data.shape[2], T, H, w.N, w.K, out.data_ptr(), out.stride(0),
                                    out.stride(1), _p(gate), gate.stride(0) if gate is not None else 0, _stream(x)),
          "cfc_head_linear")
    return out


def latent_norm(part, nq: int, wq, wc, eps: float, slots, cache, dtype) -> torch.Tensor:
    """part: fp32 slabs [split, T, nq + rank] of the joint down projection.  Writes the normed cached
    latent into ``cache`` [blocks, 32, RS] at ``slots``; returns the normed query latent [T, nq]."""
    T, N = part.shape[1], part.shape[2]
    RS = cache.shape[-1]
    if not part.is_cuda:
        q, c = ref.latent_norm(part, nq, wq, wc, eps)
        cache.view(-1, RS)[slots.long(), :N - nq] = c.to(cache.dtype)
        return q.to(dtype)
    _req(part, torch.float32, "part")
    _req(slots, torch.int32, "slots")
    if cache.dtype != dtype:
        raise TypeError(f"latent cache {cache.dtype}, activations {dtype}")
    out = torch.empty(T, nq, dtype=dtype, device=part.device)
    check(kernels().cfc_latent_norm(_act(dtype), part.data_ptr(), part.shape[0], T, nq, N - nq, wq.data_ptr(),
                                    wc.data_ptr(), float(eps), slots.data_ptr(), out.data_ptr(), nq, cache.data_ptr(), RS,
                                    _stream(part)), "cfc_latent_norm")
    return out


@dataclasses.dataclass
class Rope:
    """Rotary positions on neighbouring pairs of ``2 len(freq)`` dimensions: angle = position * freq, cos and sin
    times ``mag``."""
    freq: torch.Tensor            # fp32
    mag: float

    @property
    def dims(self) -> int:
        return 2 * self.freq.numel()


def yarn_rope(dims: int, base: float, scaling: dict | None, device) -> Rope:
    """Frequencies base^(-2i / dims); with ``scaling`` (factor, original, fast, slow) those of slow dimensions divided
    by the factor, a linear ramp between, and the length's magnitude on cos and sin."""
    i = np.arange(dims // 2, dtype=np.float64)
    f, mag = base ** (-2.0 * i / dims), 1.0
    if scaling:
        at = [dims * math.log(scaling["original"] / (2 * math.pi * scaling[k])) / (2 * math.log(base)) for k in ("fast", "slow")]
        lo, hi = max(math.floor(at[0]), 0), min(math.ceil(at[1]), dims - 1)
        ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
        f = f / scaling["factor"] * ramp + f * (1.0 - ramp)
        mag = 0.1 * math.log(scaling["factor"]) + 1.0
    return Rope(torch.tensor(f, dtype=torch.float32, device=device), mag)


def latent_rope(kv: Cols, rank: int, wc, eps: float, slots, cache, q: Cols, heads: int, dim: int, rope: Rope, positions, qr,
                vdim: int = 0, gate: Cols | None = None):
    """The normed latent (``rank`` columns of ``kv``) and the rotated shared key part behind it into ``cache``
    [blocks, 32, RS] at ``slots``; each head's rotated query part into ``qr`` [T, heads, >= rot] (heads at an even
    stride; the pad zeroed).  ``q`` columns per head [dim | rot].  Returns (unrotated queries [T, heads, dim], output gate's pre-activations
    [T, heads vdim] or None) as activations."""
    T, RS, RV, dt = qr.shape[0], cache.shape[-1], padded_rank(rank), qr.dtype
    if not qr.is_cuda:
        y = kv.value()
        c = y[:, :rank]
        c = c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * wc
        rows = cache.view(-1, RS)
        rows[slots.long(), :rank] = c.to(dt)
        rows[slots.long(), RV:RV + rope.dims] = ref.rotate_pairs(y[:, rank:], positions, rope.freq, rope.mag).to(dt)
        qv = q.value().view(T, heads, dim + rope.dims)
        qr.zero_()
        qr[:, :, :rope.dims] = ref.rotate_pairs(qv[:, :, dim:], positions, rope.freq, rope.mag).to(dt)
        return qv[:, :, :dim].to(dt), gate.value().to(dt) if gate is not None else None
    if cache.dtype != dt or qr.stride(2) != 1 or qr.stride(0) != heads * qr.stride(1) or qr.shape[1] != heads \
            or q.n != heads * (dim + rope.dims):
        raise ValueError(f"latent_rope: qr {tuple(qr.shape)} {dt}, cache rows of {RS} {cache.dtype}, {q.n} query columns")
    for name, t in (("slots", slots), ("positions", positions)):
        _req(t, torch.int32, name)
    qn = torch.empty(T, heads, dim, dtype=dt, device=qr.device) if q.slabs else None
    gt = torch.empty(T, heads * vdim, dtype=dt, device=qr.device) if gate is not None and gate.slabs else None
    g = gate.args(dt) if gt is not None else [None, 0, 0, 0]
    check(kernels().cfc_latent_rope(_act(dt), *kv.args(dt), T, rank, wc.data_ptr(), float(eps), slots.data_ptr(),
                                    cache.data_ptr(), RS, RV, *q.args(dt), heads, dim, qr.data_ptr(), qr.stride(1),
                                    qr.shape[2], _p(qn), *g, vdim, _p(gt), rope.freq.data_ptr(), rope.dims, float(rope.mag),
                                    positions.data_ptr(), _stream(qr)),
          "cfc_latent_rope")
    if qn is None:
        qn = q.t[:, q.c0:q.c0 + q.n].unflatten(1, (heads, dim + rope.dims))[:, :, :dim]
    if gate is not None and gt is None:
        gt = gate.t[:, gate.c0:gate.c0 + gate.n]
    return qn, gt


def rows_per_tile(dtype, RS: int, decode_plan: tuple | None = None, RV: int | None = None) -> int:
    """(token, head) rows of one attention work item: the general kernel's 4, or 16 / 32 / 64 on MFMA."""
    if dtype != torch.bfloat16 or (RV or RS) > MFMA_MAX_RANK or RS > MFMA_MAX_KEY:
        return ANY_ROWS
    return decode_plan[0] if decode_plan else most_rows(RS)


def most_rows(RS: int) -> int:
    """Rows of the largest work item whose registers hold: longer rows leave room for 32."""
    return 64 if RS <= MFMA_MAX_RANK else 32


MAX_PARTITIONS = 256
_TILE_US = {16: 1.8, 32: 2.1, 64: 3.9}     # one 64-key tile at rank 512, by rows per work item (one workgroup alone)


def decode_plan(B: int, heads: int, RS: int, max_ctx: int, P: int | None = None) -> tuple[int, int]:
    """(rows per work item, key slices) of a decode step, from the time of its longest workgroup plus the
    slices' partials (written and merged in fp32) against the time to stream the latents, which
    workgroups of one sequence each read: measured per-tile times, one MI355X (64-key tiles)."""
    scale = max(0.35, RS / 512)
    per_cu = max(1, min(4, (160 * 1024) // (2 * 64 * 64 * math.ceil(RS / 64) * 2 + 12 * 1024)))
    nt, best = max(1, math.ceil(max_ctx / 64)), None
    cand = [P] if P else sorted({p for p in (1, 2, 3, 4, 5, 6, 8, 10, 12, 16, 20, 24, 32, 48, 64, 96, 128) if p <= nt})
    for rows in (16, 32, 64):
        if rows > 16 and (rows >= 2 * heads or rows > most_rows(RS)):
            continue
        g = math.ceil(heads / rows)
        for p in cand:
            rounds = math.ceil(B * g * p / (256 * per_cu))
            us = _TILE_US[rows] * scale * (1.15 if rows > 16 and RS > MFMA_MAX_RANK else 1.0)
            t = max(rounds * (4 + math.ceil(nt / p) * us * min(per_cu, math.ceil(B * g * p / 256))),
                    B * max_ctx * RS * 2 * g / 7e6)
            if p > 1:
                t += 8 + 2 * B * heads * p * RS * 4 / 5e6
            if best is None or t < best[0]:
                best = (t, rows, p)
    return best[1], best[2]


def attn_tiles(cu_q, heads: int, rows: int, ctx_lens=None, window: int = 0):
    """(sequence, first row) of every work item of a packed batch; with ``ctx_lens`` those with the most
    keys (at most about ``window``) first, so the long ones do not end the grid alone."""
    tiles = []
    for s in range(len(cu_q) - 1):
        n = cu_q[s + 1] - cu_q[s]
        base = ctx_lens[s] - n if ctx_lens is not None else 0
        for m0 in range(0, n * heads, rows):
            keys = base + (min(m0 + rows, n * heads) - 1) // heads
            tiles.append((min(keys, window) if window else keys, s, m0))
    if ctx_lens is not None:
        tiles.sort(key=lambda t: -t[0])
    return [t[1] for t in tiles], [t[2] for t in tiles]


def partitions(n_tiles: int, max_ctx: int, target: int = 512) -> int:
    """Key slices per work item: enough workgroups to fill the chip, at least four 64-key tiles each."""
    return max(1, min(math.ceil(target / max(1, n_tiles)), math.ceil(max_ctx / 256), MAX_PARTITIONS))


def latent_attention(q, cache, block_tables, cu_q, ctx_lens, scale: float, tiles=None, rows: int | None = None,
                     P: int = 1, workspace=None, window: int = 0, sink=None, RV: int | None = None) -> torch.Tensor:
    """Softmax attention of q [T, H, RS] over the paged rows [blocks, 32, RS], causal inside each sequence's
    portion; the value is a row's first ``RV`` columns (None: all).  ``window``: keys a token sees, itself included
    (0: all before it).  ``sink`` [H] fp32: exp(sink) joins each denominator once.  ``cu_q`` None: one token per
    sequence.  ``tiles``: device (tile_seq, tile_m0) of :func:`attn_tiles` cut for ``rows``; P key slices per tile
    merged at the end."""
    T, H, RS = q.shape
    RV = RV or RS
    B = ctx_lens.numel()
    if not q.is_cuda:
        cu = cu_q if cu_q is not None else torch.arange(B + 1)
        return ref.latent_attention(q, cache, block_tables, cu, ctx_lens, scale, window, sink, RV)
    if not q.is_contiguous() or not cache.is_contiguous() or cache.shape[-1] != RS or cache.dtype != q.dtype:
        raise ValueError(f"latent_attention: q {tuple(q.shape)} {q.dtype}, cache {tuple(cache.shape)} {cache.dtype}")
    for name, t in (("block_tables", block_tables), ("ctx_lens", ctx_lens)):
        _req(t, torch.int32, name)
    rows = rows or rows_per_tile(q.dtype, RS, decode_plan(B, H, RS, 64, P) if cu_q is None else None, RV)
    if cu_q is None:
        if T != B:
            raise ValueError(f"latent_attention: {T} rows for {B} sequences")
        per_seq = math.ceil(H / rows)
        ts = tm = None
        n_tiles = B * per_seq
    else:
        if tiles is None:
            a, b = attn_tiles(cu_q.tolist(), H, rows, ctx_lens.tolist())
            tiles = tuple(torch.tensor(v, dtype=torch.int32, device=q.device) for v in (a, b))
        ts, tm = tiles
        per_seq, n_tiles = 0, ts.numel()
    if sink is not None:
        _req(sink, torch.float32, "sink")
    out = torch.empty(T, H, RV, dtype=q.dtype, device=q.device)
    po = pm = None
    if P > 1:
        need = T * H * P * (RV + 2)
        ws = workspace if workspace is not None and workspace.numel() >= need else _workspace(q.device, need)
        po, pm = ws[:T * H * P * RV], ws[T * H * P * RV:need]
    check(kernels().cfc_latent_attention(_act(q.dtype), q.data_ptr(), cache.data_ptr(), block_tables.data_ptr(), _p(cu_q),
                                         ctx_lens.data_ptr(), _p(ts), _p(tm), n_tiles, per_seq, rows, H, RS, RV,
                                         block_tables.shape[1], float(scale), int(window), _p(sink), P, T * H, _p(po), _p(pm), out.data_ptr(),
                                         _stream(q)), "cfc_latent_attention")
    return out


# ------------------------------------------------------- long portions: expanded keys and values
EXPANDED_DIM = 128        # head size of the prefill attention kernel
ROT_COLS = 64             # columns of its second key part


def gather_tiles(ctx_lens, starts=None) -> tuple[list, list]:
    """Dense layout of sequences (from the 64-token tile of position ``starts[s]`` on), 64-token tiles: ([(sequence,
    first position)], row of position 0 per sequence -- negative where the layout starts later)."""
    tiles, base, n = [], [], 0
    for s, ctx in enumerate(ctx_lens):
        lo, hi = starts[s] // 64 if starts is not None else 0, -(-ctx // 64)
        base.append(n - 64 * lo)
        tiles += [(s, 64 * i) for i in range(lo, hi)]
        n += 64 * (hi - lo)
    return tiles, base


def expand(cache, block_tables, ctx_lens, tiles, uk, uv, RV: int | None = None):
    """Keys [tokens, H * 128] and transposed, slot-ordered values [H * 128, tokens] (row stride padded) of the
    sequences of ``tiles`` (:func:`gather_tiles`): uk a PackedWeight [H * 128, RV], uv row-major [H * 128, RV].  ``RV``:
    latent columns of a row, where a rotated key part follows: it comes third, [tokens, 64]."""
    from . import kernels as K
    n, RS = tiles.shape[0], cache.shape[-1]
    k2 = torch.empty(n * 64, ROT_COLS, dtype=cache.dtype, device=cache.device) if RV is not None else None
    RV = RV or RS
    rows = torch.empty(2, n * 64, RV, dtype=cache.dtype, device=cache.device)
    check(kernels().cfc_latent_gather(cache.data_ptr(), block_tables.data_ptr(), block_tables.shape[1], ctx_lens.data_ptr(),
                                      tiles.data_ptr(), n, RS, RV, rows[0].data_ptr(), rows[1].data_ptr(), _p(k2), _stream(cache)),
          "cfc_latent_gather")
    k = K.pgemm(rows[0], uk, variant="ppp")
    # the values' rows are read side by side: an odd number of 128-byte lines apart, not a power of two
    ldv = n * 64 + (64 if n % 2 == 0 else 128)
    vt = torch.empty(uv.shape[0], ldv, dtype=cache.dtype, device=cache.device)[:, :n * 64]
    K.pgemm(uv, K.PackedWeight(rows[1].view(-1), n * 64, RV, 64), out=vt, variant="ppp")
    return (k, vt) if k2 is None else (k, vt, k2)


def expanded_attention(q, k, vt, tok_base, cu_q, ctx_lens, scale: float, tiles, out) -> torch.Tensor:
    """Causal attention of q [T, H, 128] over :func:`expand`'s keys and values into ``out`` [T, H, 128] (row stride
    free, heads dense); ``tiles``: ops.kernels.prefill_tiles for 256-row tiles."""
    T, H, D = q.shape
    if D != EXPANDED_DIM or not q.is_contiguous() or out.stride(1) != D or out.stride(2) != 1:
        raise ValueError(f"expanded_attention: q {tuple(q.shape)}, out strides {out.stride()}")
    check(kernels().cfc_prefill_attention_expanded(q.data_ptr(), k.data_ptr(), vt.data_ptr(), tok_base.data_ptr(),
                                                   vt.stride(0), cu_q.data_ptr(), ctx_lens.data_ptr(), tiles[0].data_ptr(),
                                                   tiles[1].data_ptr(), tiles[0].numel(), H, float(scale), out.data_ptr(),
                                                   out.stride(0), _stream(q)), "cfc_prefill_attention_expanded")
    return out


def expanded_window_attention(q: Cols, q2, k, k2, vt, tok_base, cu_q, ctx_lens, scale: float, tiles, window: int, sink, gate, out):
    """The same with a second key part k2 [tokens, 64] shared by all heads and the heads' q2 [T, H, 64], a sliding
    ``window`` (0: none), a ``sink`` per head and an output ``gate`` [T, H * 128].  ``q``: columns of which head h's 128
    start at h * (columns per head)."""
    T, H = q2.shape[:2]
    p, _, q_ld, _ = q.args(out.dtype)
    if q2.shape[2] != ROT_COLS or not q2.is_contiguous() or out.shape != (T, H * EXPANDED_DIM) or out.stride(1) != 1 \
            or gate.shape != out.shape or gate.stride(1) != 1:
        raise ValueError(f"expanded_window_attention: q2 {tuple(q2.shape)}, gate {tuple(gate.shape)}, out {tuple(out.shape)}")
    check(kernels().cfc_prefill_attention_expanded2(p, q_ld, q.n // H, q2.data_ptr(), k.data_ptr(), k2.data_ptr(), vt.data_ptr(),
                                                    tok_base.data_ptr(), vt.stride(0), cu_q.data_ptr(), ctx_lens.data_ptr(),
                                                    tiles[0].data_ptr(), tiles[1].data_ptr(), tiles[0].numel(), H, float(scale),
                                                    int(window), _p(sink), gate.data_ptr(), gate.stride(0), out.data_ptr(),
                                                    out.stride(0), _stream(q2)), "cfc_prefill_attention_expanded2")
    return out
