"""Real-gated linear recurrence with block-diagonal gates behind a short convolution (csrc/kernels/rglru.hip).

GPU tensors go to the native library (which must be built), CPU tensors to the fp32 reference.
"""
from __future__ import annotations

import dataclasses
import math

import torch
import torch.nn.functional as F

from . import reference as ref
from ._native import check, kernels
from .cols import Cols
from .kernels import _p, _req, _stream
from .stream import _act

SEGMENT = 128            # tokens per segment of the prompt kernels
MAX_BLOCK = 512          # block columns (padded) they take; wider ones and fp32: the general kernels


@dataclasses.dataclass
class RgLru:
    """Weights of a recurrent block between its projections: vectors fp32 [W], ``conv`` [taps, W] fp32, gate matrices ``ra``
    and ``ri`` [blocks, out, in] in the activations' dtype.  ``rate`` <= 0: log of the decay with the gate fully open."""
    bx: torch.Tensor
    conv: torch.Tensor
    cb: torch.Tensor
    ra: torch.Tensor
    ra_b: torch.Tensor
    ri: torch.Tensor
    ri_b: torch.Tensor
    rate: torch.Tensor
    by: torch.Tensor

    def __post_init__(self):
        self.blocks, self.bs, _ = self.ra.shape
        self.f32 = self.ra.dtype == torch.float32
        if self.ra.shape[1] != self.ra.shape[2] or self.ri.shape != self.ra.shape or self.width != self.bx.numel():
            raise ValueError(f"gates {tuple(self.ra.shape)}, {tuple(self.ri.shape)} for a width of {self.bx.numel()}")
        if self.f32:
            self.KP, self.NP = 4 * math.ceil(self.bs / 4), self.bs
            self.packed = torch.stack([self.ra, self.ri]).transpose(2, 3).contiguous()      # [2, blocks, in, out]
        else:
            self.KP, self.NP = 32 * math.ceil(self.bs / 32), 16 * math.ceil(self.bs / 16)
            self.packed = F.pad(torch.stack([self.ra, self.ri]), (0, self.KP - self.bs, 0, self.NP - self.bs)).contiguous()
        if self.ra.is_cuda:
            self.ra = self.ri = None                 # the packed copy serves

    @property
    def width(self) -> int:
        return self.blocks * self.bs

    @property
    def taps(self) -> int:
        return self.conv.shape[0]

    @property
    def ring(self) -> int:
        """Rows of a sequence's convolution state."""
        return self.taps

    def nbytes(self) -> int:
        return self.packed.numel() * self.packed.element_size()

    def weights(self) -> list:
        return [self.bx.data_ptr(), self.conv.data_ptr(), self.cb.data_ptr(), self.taps, self.ra_b.data_ptr(), self.ri_b.data_ptr(),
                self.rate.data_ptr(), self.by.data_ptr(), self.packed.data_ptr(), self.blocks, self.bs, self.KP, self.NP]


def _ref(p: RgLru, x, y, slots, positions, cu, tail, state, out):
    """``positions``: of each portion's first row."""
    X, Y, taps = x.value(), y.value(), p.taps
    for s, slot in enumerate(slots.tolist()):
        a, b, pos0 = int(cu[s]), int(cu[s + 1]), int(positions[s])
        if pos0 == 0:
            state[slot].zero_()
        past = [tail[slot, q % p.ring] + p.bx if q >= 0 else torch.zeros(p.width) for q in range(pos0 - taps + 1, pos0)]
        ext = torch.cat([torch.stack(past), X[a:b] + p.bx]) if past else X[a:b] + p.bx
        u = (p.cb + sum(p.conv[j] * ext[j:j + b - a] for j in range(taps))).to(out.dtype).float()
        for r in range(max(a, b - taps + 1), b):
            tail[slot, (pos0 + r - a) % p.ring] = X[r]
        ub = u.view(b - a, p.blocks, p.bs).transpose(0, 1)
        pr, pi = (torch.matmul(ub, w.float().transpose(1, 2)).transpose(0, 1).reshape(b - a, -1) for w in (p.ra, p.ri))
        S = ref.rglru(u, pr + p.ra_b, pi + p.ri_b, p.rate, state[slot])
        out[a:b] = (S * ref.gelu_tanh(Y[a:b] + p.by)).to(out.dtype)
    return out


def whole_portions(cu, width: int) -> bool:
    """Whether the portions of a pass are one segment each.  That takes as long as the longest one's tokens in turn; segments
    take launches and two passes over all elements (microseconds measured on one MI355X)."""
    return 0.1 * max(b - a for a, b in zip(cu, cu[1:])) <= 25.0 + 5.7e-6 * (cu[-1] - cu[0]) * width


def _fits(p: RgLru, x: Cols, y: Cols, tail, state, out):
    if x.n != p.width or y.n != p.width or out.shape != (x.rows, p.width) or not out.is_contiguous() or state.shape[-1] != p.width \
            or tail.shape[1:] != (p.ring, p.width) or p.f32 != (out.dtype == torch.float32):
        raise ValueError(f"rglru: columns {x.n}, {y.n}, state {tuple(state.shape)}, tail {tuple(tail.shape)}, out {tuple(out.shape)} "
                         f"{out.dtype} for a width of {p.width}")
    _req(tail, torch.float32, "tail")
    _req(state, torch.float32, "state")
    return x.args(out.dtype), y.args(out.dtype)


def step(p: RgLru, x: Cols, y: Cols, slots, positions, ctx_lens, tail, state, out) -> torch.Tensor:
    """One token per sequence: S gelu(y) into ``out`` [B, W]; ``state`` [slots, W] and the convolution's inputs ``tail``
    [slots, ring, W] fp32 are updated."""
    if not out.is_cuda:
        return _ref(p, x, y, slots, positions, torch.arange(len(slots) + 1), tail, state, out)
    for name, t in (("slots", slots), ("positions", positions), ("ctx_lens", ctx_lens)):
        _req(t, torch.int32, name)
    xa, ya = _fits(p, x, y, tail, state, out)
    check(kernels().cfc_rglru_step(int(p.f32), *xa, *ya, *p.weights(), tail.data_ptr(), state.data_ptr(), slots.data_ptr(),
                                   positions.data_ptr(), ctx_lens.data_ptr(), out.shape[0], out.data_ptr(), _stream(out)), "cfc_rglru_step")
    return out


def prefill(p: RgLru, x: Cols, y: Cols, slots, cu_q, ctx_lens, tiles, chunks, chunk_cu, tail, state, out) -> torch.Tensor:
    """Packed portions, ``x`` and ``y`` activations; ``tiles`` of ops.stream.conv_tiles (by rows), ``chunks`` and ``chunk_cu``
    of ops.gru.chunk_plan with SEGMENT, on the device; both None: every portion is one segment (:func:`whole_portions`)."""
    if not out.is_cuda:
        first = ctx_lens - (cu_q[1:] - cu_q[:-1])
        return _ref(p, x, y, slots, first, cu_q, tail, state, out)
    whole = chunks is None
    for name, t in (("slots", slots), ("cu_q", cu_q), ("ctx_lens", ctx_lens), ("tiles", tiles)) + \
            (() if whole else (("chunks", chunks), ("chunk_cu", chunk_cu))):
        _req(t, torch.int32, name)
    xa, ya = _fits(p, x, y, tail, state, out)
    if xa[1] or ya[1]:
        raise ValueError("rglru prefill: x and y are activations")
    T, n, mfma = out.shape[0], 0 if whole else chunks.shape[0], not p.f32 and p.KP <= MAX_BLOCK
    u = torch.empty(T, p.blocks * p.KP, dtype=out.dtype, device=out.device)
    sums = None if mfma and whole else torch.empty((n if mfma else T) * 2 * p.width, dtype=torch.float32, device=out.device)
    check(kernels().cfc_rglru_prefill(_act(out.dtype), xa[0], xa[2], ya[0], ya[2], *p.weights(), tail.data_ptr(), state.data_ptr(),
                                      slots.data_ptr(), tiles.data_ptr(), tiles.shape[1], int(whole), _p(chunks), n, _p(chunk_cu),
                                      cu_q.data_ptr(), ctx_lens.data_ptr(), slots.numel(), T, u.data_ptr(), _p(sums),
                                      out.data_ptr(), _stream(out)), "cfc_rglru_prefill")
    return out
