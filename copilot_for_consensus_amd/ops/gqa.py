"""Grouped-query attention over two key ranges: a sliding window or the own chunk of positions, and either kept first
tokens or mean keys and values of earlier blocks; scores with a softcap and a bias by distance, outputs through a gate
(csrc/kernels/qkv.hip, gqa.hip).

GPU tensors go to the native library (which must be built), CPU tensors to the fp32 reference.
"""
from __future__ import annotations

import bisect
import dataclasses
import math
from fractions import Fraction

import numpy as np
import torch

from . import reference as ref
from ._native import check, kernels
from .cols import Cols
from .kernels import _p, _req, _stream, _workspace
from .stream import _act

KV_BLOCK = ref.KV_BLOCK
MFMA_DIMS = (32, 64, 96, 128, 160, 192, 256)      # head columns the MFMA kernels are built for
MAX_DIM = 1024
ANY_ROWS = 4              # rows per tile of the general kernel
MAX_PARTITIONS = 256
LOG2E = 1.4426950408889634
CAP_NEAR = (0.25, 0.35)   # scores up to these shares of their cap take shorter forms of the cap


@dataclasses.dataclass(frozen=True)
class Mask:
    """What a token sees: its last ``size`` tokens (0: all), or with ``chunked`` those of its own run of ``size`` positions
    (counted from 0), the first ``keep``, one mean per block of ``pool`` tokens wholly ahead of the window (0: none)."""
    size: int
    keep: int = 0
    pool: int = 0
    chunked: bool = False

    def __post_init__(self):
        if min(self.size, self.keep, self.pool) < 0 or (self.pool and (self.keep or not self.size)):
            raise ValueError(f"{self}: pooled blocks need a window and no kept tokens")
        if self.chunked and (not self.size or self.pool):
            raise ValueError(f"{self}: chunks have a size and no pooled blocks")

    def visible(self, ctx: int) -> int:
        """Keys and means the last of ``ctx`` tokens sees (about)."""
        if not self.size or ctx <= self.size:
            return ctx
        return self.size + (ctx - self.size) // self.pool if self.pool else min(ctx, self.size + self.keep)


def padded_dim(dim: int, vdim: int) -> int:
    """Columns of a cached head: a size the MFMA kernels take where one fits, the pad zero."""
    d = max(dim, vdim)
    return next((m for m in MFMA_DIMS if m >= d), 32 * math.ceil(d / 32))


def pool_entries(pool: int) -> int:
    """Entries per cache block for the means of blocks of ``pool`` tokens: a power of two with entries * pool >= 32, so
    that entry b's cache block exists once token block b is complete."""
    return 1 << math.ceil(math.log2(KV_BLOCK / pool)) if pool < KV_BLOCK else 1


def distance_starts(rows: int, far) -> list[int]:
    """First distance of each of a bias table's ``rows`` rows: one distance each in the first half, then steps of equal
    ratio, the last row's one step short of ``far``: n is at or past the k-th when (n / half)^steps >= (far / half)^k."""
    half = rows // 2
    if rows < 2:
        return [0] * rows
    far = Fraction(far)
    if far <= half:
        raise ValueError(f"distance bias of {rows} rows up to a distance of {far}")
    steps, out = rows - half, list(range(half + 1))
    for k in range(1, steps):
        n, level = math.floor(half * (float(far) / half) ** (k / steps)), far ** k * half ** (steps - k)
        while n ** steps >= level:
            n -= 1
        while n ** steps < level:
            n += 1
        out.append(n)
    return out


def distance_bias(rel: torch.Tensor, far, limit: int) -> torch.Tensor:
    """[H, n] biases by distance from a table ``rel`` [rows, H] (:func:`distance_starts`), the last entry for all distances
    from there on; no more than ``limit`` (> 0) distances."""
    starts = distance_starts(rel.shape[0], far)
    n = starts[-1] + 1
    row = [bisect.bisect_right(starts, d) - 1 for d in range(min(n, limit) if limit else n)]
    return rel.float()[torch.tensor(row, dtype=torch.long, device=rel.device)].t().contiguous()


@dataclasses.dataclass
class Heads:
    """An attention layer between its projections and its output: ``H`` query heads in ``G`` groups.  Norm weights over the
    whole projection ([H dim], [G dim]) or per head ([dim]), fp32; ``conv`` [taps, (H + G) dim + G vdim] fp32 over time
    ahead of the norms; ``freq`` the rotation of the first dimensions.  ``shared``: keys and values are another layer's.
    ``softcap`` of the scores (0: none), then ``bias`` [H, n] fp32 by distance (:func:`distance_bias`).  ``unit``: norms per
    head with weights of 1, so that no score exceeds ``dim * scale``."""
    H: int
    G: int
    dim: int
    vdim: int
    scale: float
    mask: Mask
    eps: float
    q_norm: torch.Tensor | None
    k_norm: torch.Tensor | None
    per_head: bool
    sink: torch.Tensor | None
    freq: torch.Tensor | None = None
    conv: torch.Tensor | None = None
    shared: bool = False
    softcap: float = 0.0
    bias: torch.Tensor | None = None
    unit: bool = False

    def __post_init__(self):
        self.D = padded_dim(self.dim, self.vdim)
        # queries carry the scale into the softmax's base 2, or into the cap's e^(2 score / cap)
        self.q_scale = self.scale * LOG2E * (2.0 / self.softcap if self.softcap else 1.0)
        share = 1.02 * self.dim * abs(self.scale) / self.softcap if self.unit and self.softcap else 1.0
        self.capped = 0 if not self.softcap else 3 if share <= CAP_NEAR[0] else 2 if share <= CAP_NEAR[1] else 1
        self.bias2 = None if self.bias is None else (self.bias * LOG2E).contiguous()
        if self.bias is not None and (self.bias.shape[0] != self.H or self.mask.pool):
            raise ValueError(f"bias {tuple(self.bias.shape)} for {self.H} heads over {self.mask}")
        if self.H % self.G or self.D > MAX_DIM:
            raise ValueError(f"{self.H} heads in {self.G} groups, {self.D} columns")

    @property
    def taps(self) -> int:
        return 1 if self.conv is None else self.conv.shape[0]

    @property
    def columns(self) -> int:
        """Columns of the projections' product."""
        return self.H * self.dim + (0 if self.shared else self.G * (self.dim + self.vdim))


def rope_freq(dims: int, base: float, device) -> torch.Tensor | None:
    """base^(-2i / dims), in fp32."""
    if not dims:
        return None
    f = base ** (-2.0 * np.arange(dims // 2, dtype=np.float64) / dims)
    return torch.tensor(f, dtype=torch.float32, device=device)


def qkv_rows(a: Heads, cols: Cols, rows, positions, slots, states, block_tables, tail=None, lead=None) -> torch.Tensor:
    """Projections [q | k | v] of packed rows to queries [T, H, D] (scaled by ``q_scale``) and rows of the cache ``rows``
    (runtime.kv_cache.PagedHeads) at ``slots``.  ``lead``: rows of the same portion before each row (prompts: afterwards
    :func:`conv_tail` and :func:`pool_rows`); None: one token per sequence, whose state in ``tail`` [states, taps - 1, C]
    and pooled entries are written here."""
    T, dt = cols.rows, rows.k.dtype
    if cols.n != a.columns or rows.k.shape[1] != a.G or rows.k.shape[3] != a.D:
        raise ValueError(f"qkv_rows: {cols.n} columns of {a.columns}, cache {tuple(rows.k.shape)}")
    if not rows.k.is_cuda:
        return _qkv_ref(a, cols, rows, positions, slots, states, block_tables, tail, lead, dt)
    for name, t in (("positions", positions), ("slots", slots)):
        _req(t, torch.int32, name)
    q = (torch.empty if a.D == a.dim else torch.zeros)(T, a.H, a.D, dtype=dt, device=rows.k.device)
    rot = 2 * a.freq.numel() if a.freq is not None else 0
    check(kernels().cfc_qkv_rows(_act(dt), *cols.args(dt), T, a.H, a.G, a.dim, a.vdim, a.D, 1 if a.shared else 3, _p(a.q_norm),
                                 _p(a.k_norm), int(a.per_head), float(a.eps), _p(a.freq), rot, float(a.q_scale), _p(a.conv),
                                 a.taps, _p(tail), _p(lead), _p(states), positions.data_ptr(), slots.data_ptr(), q.data_ptr(),
                                 rows.k.data_ptr(), rows.v.data_ptr(), _p(rows.pk), _p(rows.pv), a.mask.pool, rows.log2_entries,
                                 block_tables.data_ptr(), block_tables.shape[1], _stream(q)), "cfc_qkv_rows")
    return q


def _qkv_ref(a, cols, rows, positions, slots, states, block_tables, tail, lead, dt):
    T, u = cols.rows, cols.value()
    first = lead is None
    lead = torch.zeros_like(positions) if first else lead
    if a.conv is not None:
        y = ref.conv_over_time(u, a.conv, lead, positions, states, tail)
        if first and a.taps > 1:
            for t, (s, p) in enumerate(zip(states.tolist(), positions.tolist())):
                tail[s, p % (a.taps - 1)] = u[t]
        u = y
    nq, nk = a.H * a.dim, a.G * a.dim

    def turned(x, w, heads):
        x = (ref.head_norm(x, w, a.eps, a.per_head, heads) if w is not None else x).view(T, heads, a.dim)
        return ref.rotate_heads(x, positions, a.freq) if a.freq is not None else x
    q = torch.zeros(T, a.H, a.D, dtype=dt)
    q[..., :a.dim] = (turned(u[:, :nq], a.q_norm, a.H) * a.q_scale).to(dt)
    if a.shared:
        return q
    blk, off = (slots // KV_BLOCK).long(), (slots % KV_BLOCK).long()
    rows.k[blk, :, off, :a.dim] = turned(u[:, nq:nq + nk], a.k_norm, a.G).to(dt)
    rows.v[blk, :, off, :a.vdim] = u[:, nq + nk:].reshape(T, a.G, a.vdim).to(dt)
    if first and a.mask.pool:
        done = [(t, p // a.mask.pool) for t, p in enumerate(positions.tolist()) if (p + 1) % a.mask.pool == 0]
        pool_rows(a, rows, torch.tensor(done, dtype=torch.int32).reshape(-1, 2), block_tables)
    return q


def conv_tail(a: Heads, cols: Cols, cu_q, ctx_lens, states, tail) -> None:
    """The last inputs of each portion's convolution into the sequences' state."""
    if a.taps < 2:
        return
    if not tail.is_cuda:
        u = cols.value()
        for s, slot in enumerate(states.tolist()):
            lo, hi, ctx = int(cu_q[s]), int(cu_q[s + 1]), int(ctx_lens[s])
            for d in range(min(a.taps - 1, hi - lo)):
                tail[slot, (ctx - 1 - d) % (a.taps - 1)] = u[hi - 1 - d]
        return
    p, split, ld, plane = cols.args()
    check(kernels().cfc_conv_tail(int(not cols.slabs and cols.t.dtype == torch.float32), p, split, ld, plane, cols.n, cu_q.data_ptr(),
                                  ctx_lens.data_ptr(), states.data_ptr(), states.numel(), a.taps, tail.data_ptr(), _stream(tail)),
          "cfc_conv_tail")


def ended_blocks(cu, ctx, pool: int) -> np.ndarray:
    """[n, 2] (portion, block) of every block of ``pool`` tokens whose last token lies in the packed portions."""
    out = [(s, b) for s, (lo, hi, c) in enumerate(zip(cu, cu[1:], ctx)) for b in range((c - (hi - lo)) // pool, c // pool)]
    return np.asarray(out, np.int32).reshape(-1, 2)


def pool_rows(a: Heads, rows, blocks, block_tables) -> None:
    """Mean keys and values of ``blocks`` (:func:`ended_blocks` on the device) into the pooled cache."""
    if not blocks.shape[0]:
        return
    P, e = a.mask.pool, rows.pk.shape[2] if rows.pk is not None else 0
    if not rows.k.is_cuda:
        for s, b in blocks.tolist():
            page, at = int(block_tables[s, b // e]), b % e
            for c, pc in ((rows.k, rows.pk), (rows.v, rows.pv)):
                own = [c[int(block_tables[s, p // KV_BLOCK]), :, p % KV_BLOCK].float() for p in range(b * P, b * P + P)]
                pc[page, :, at] = (sum(own) / P).to(pc.dtype)
        return
    _req(blocks, torch.int32, "blocks")
    check(kernels().cfc_pool_rows(_act(rows.k.dtype), blocks.data_ptr(), blocks.shape[0], block_tables.data_ptr(), block_tables.shape[1],
                                  rows.k.data_ptr(), rows.v.data_ptr(), rows.pk.data_ptr(), rows.pv.data_ptr(), a.G, a.D, P,
                                  rows.log2_entries, _stream(rows.k)), "cfc_pool_rows")


def prompt_rows(dtype, D: int) -> int:
    """Rows of a prompt tile (per key head), 0: the general kernel's tiles over all heads."""
    return (256 if D in (64, 128) else 128) if dtype == torch.bfloat16 and D in MFMA_DIMS else 0


def prompt_tiles(cu, ctx, H: int, G: int, rows: int) -> np.ndarray:
    """[2, n] (sequence, first row) of the tiles of packed portions, the latest positions (most keys) first."""
    per, step = (H // G, rows) if rows else (H, ANY_ROWS)
    seq, m0, pos = [], [], []
    for s, (lo, hi, c) in enumerate(zip(cu, cu[1:], ctx)):
        m = np.arange(0, (hi - lo) * per, step)
        seq.append(np.full(len(m), s))
        m0.append(m)
        pos.append(c - (hi - lo) + np.minimum(m + step, (hi - lo) * per) // per)
    order = np.argsort(-np.concatenate(pos), kind="stable")
    return np.stack([np.concatenate(seq)[order], np.concatenate(m0)[order]]).astype(np.int32)


def decode_slices(B: int, H: int, G: int, D: int, visible: int, dtype) -> int:
    """Key slices per row of a decode step: about four workgroups per CU, at least eight 32-key tiles each."""
    if dtype != torch.bfloat16 or D not in MFMA_DIMS:
        return max(1, min(math.ceil(1024 / (B * math.ceil(H / ANY_ROWS))), visible // 256, MAX_PARTITIONS))
    items = B * G * math.ceil(H / G / 16)
    return max(1, min(math.ceil(1024 / items), visible // 256, MAX_PARTITIONS))


def attention(a: Heads, q, rows, block_tables, ctx_lens, cu_q=None, tiles=None, P: int = 1, workspace=None, gate: Cols | None = None,
              factor: float = 1.0, out: torch.Tensor | None = None) -> torch.Tensor:
    """Attention of :func:`qkv_rows`' queries over the paged rows: [T, H vdim].  ``cu_q`` None: one token per sequence, P key
    slices each; else packed portions with ``tiles`` of :func:`prompt_tiles` (on the device).  ``gate`` [T, H vdim]: the
    result times factor sigmoid(gate).  ``out``: where to (row-strided)."""
    T, H, D = q.shape
    m, dt = a.mask, q.dtype
    B = ctx_lens.numel()
    if not q.is_cuda:
        cu = cu_q if cu_q is not None else torch.arange(B + 1)
        y = ref.grouped_attention(q, rows.k, rows.v, (rows.pk, rows.pv), block_tables, cu, ctx_lens, m.size, m.keep, m.pool,
                                  a.sink, a.vdim, m.chunked, a.softcap, a.bias)
        y = y * factor * torch.sigmoid(gate.value()) if gate is not None else y * factor
        return y.to(dt) if out is None else out.copy_(y)
    if not q.is_contiguous() or rows.k.shape[1] != a.G or rows.k.shape[3] != D or rows.k.dtype != dt or H != a.H \
            or (m.pool and (rows.pk is None or rows.pool != m.pool)):
        raise ValueError(f"attention: q {tuple(q.shape)} {dt}, cache {tuple(rows.k.shape)} {rows.k.dtype}, {m}")
    for name, t in (("block_tables", block_tables), ("ctx_lens", ctx_lens)):
        _req(t, torch.int32, name)
    if a.sink is not None:
        _req(a.sink, torch.float32, "sink")
    mfma = prompt_rows(dt, D)
    if cu_q is None:
        if T != B:
            raise ValueError(f"attention: {T} rows for {B} sequences")
        kind, ts, tm, n = (1, None, None, 0) if mfma else (0, None, None, B * math.ceil(H / ANY_ROWS))
    else:
        kind, P = 2 if mfma else 0, 1
        _req(cu_q, torch.int32, "cu_q")
        _req(tiles, torch.int32, "tiles")
        ts, tm, n = tiles[0], tiles[1], tiles.shape[1]
    if gate is not None and (gate.n != H * a.vdim or gate.rows != T):
        raise ValueError(f"attention: gate of {gate.n} columns and {gate.rows} rows for {T} x {H * a.vdim}")
    if out is None:
        out = torch.empty(T, H * a.vdim, dtype=dt, device=q.device)
    elif out.shape != (T, H * a.vdim) or out.stride(1) != 1 or out.dtype != dt:
        raise ValueError(f"attention: out {tuple(out.shape)} {out.dtype}")
    po = pm = None
    if P > 1:
        need = T * H * P * (D + 2)
        ws = workspace if workspace is not None and workspace.numel() >= need else _workspace(q.device, need)
        po, pm = ws[:T * H * P * D], ws[T * H * P * D:need]
    check(kernels().cfc_gqa_attention(kind, _act(dt), q.data_ptr(), rows.k.data_ptr(), rows.v.data_ptr(), _p(rows.pk), _p(rows.pv),
                                      block_tables.data_ptr(), _p(cu_q), ctx_lens.data_ptr(), _p(ts), _p(tm), n, B, H, a.G, D, a.vdim,
                                      block_tables.shape[1], m.size, m.keep, m.pool, rows.log2_entries, int(m.chunked), a.capped,
                                      float(a.softcap * LOG2E), _p(a.bias2), a.bias2.shape[1] if a.bias2 is not None else 0, _p(a.sink),
                                      *(gate.args(dt) if gate is not None else (None, 0, 0, 0)), float(factor), P, T * H, _p(po),
                                      _p(pm), out.data_ptr(), out.stride(0), _stream(q)), "cfc_gqa_attention")
    return out
