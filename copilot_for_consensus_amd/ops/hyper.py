"""Hyper-connections (csrc/kernels/hyper.hip): several copies of the 32-bit stream, mixed after every sublayer, a weighted sum
of them read and normed by the next, in one pass.

GPU tensors go to the native library (which must be built), CPU tensors to the fp32 reference.
"""
from __future__ import annotations

import dataclasses

import torch

from . import reference as ref
from ._native import check, kernels
from .kernels import _p, _req, _stream
from .stream import Tail, _act

MAX_STREAMS = 16


@dataclasses.dataclass
class Connection:
    """A sublayer's weights on the streams, fp32: it reads sum_s ``inp``[s] x_s; then x_t <- sum_s ``mix``[s, t] x_s +
    ``out``[t] y."""
    inp: torch.Tensor
    mix: torch.Tensor
    out: torch.Tensor


class Streams:
    """The copies [T, S, W] fp32, at first all the same row ``e`` [T, W]."""

    def __init__(self, e: torch.Tensor, S: int):
        if not 1 <= S <= MAX_STREAMS:
            raise ValueError(f"{S} streams (1 to {MAX_STREAMS})")
        _req(e, torch.float32, "stream") if e.is_cuda else None
        self.S, self.e, self.x = S, e, None
        # (slabs [split, T, W] fp32, connection) of the sublayer that is done and not yet added
        self.done: tuple[torch.Tensor, Connection] | None = None

    def value(self) -> torch.Tensor:
        """CPU: the copies with what is pending added."""
        x = self.x if self.x is not None else self.e[:, None].expand(-1, self.S, -1)
        if self.done is not None:
            y, c = self.done
            self.x = x = ref.hyper_update(x, y.sum(0), c.mix, c.out)
            self.done = None
        return x

    def read(self, inp) -> torch.Tensor:
        x = self.value()
        return x.sum(1) if inp is None else torch.einsum("tsw,s->tw", x, inp)

    def _launch(self, mode, f32, n, rows, inp, w, eps, u, rstd, conv, positions, tail, h, store):
        T, W = self.e.shape
        src, ldx, lds = (self.e, W, 0) if self.x is None else (self.x, self.S * W, W)
        y = mix = out = dst = None
        if self.done is not None:
            y, c = self.done
            mix, out = c.mix, c.out
            _req(y, torch.float32, "y")
            if y.shape[1:] != (T, W) or mix.shape != (self.S, self.S) or not y.is_contiguous() or not mix.is_contiguous():
                raise ValueError(f"hyper_norm: y {tuple(y.shape)}, mix {tuple(mix.shape)} for {self.S} streams of {T} x {W}")
            if store and self.x is None:
                self.x = torch.empty(T, self.S, W, dtype=torch.float32, device=self.e.device)
            dst = self.x if store else None
        ring, slots = (tail.rows.shape[1], tail.block_tables) if tail is not None and tail.rows is not None else (0, None)
        check(kernels().cfc_hyper_norm(mode, f32, n, _p(rows), src.data_ptr(), ldx, lds, _p(dst), _p(y), y.shape[0] if y is not None else 0,
                                       _p(mix), _p(out), _p(inp), _p(w), float(eps), T, W, self.S, _p(u), _p(rstd), _p(conv),
                                       conv.shape[0] if conv is not None else 1, _p(positions), _p(slots),
                                       tail.rows.data_ptr() if ring else None, ring, _p(h), _stream(src)), "cfc_hyper_norm")
        if store:
            self.done = None


def stats(xs: Streams, inp, eps: float, u, rstd) -> None:
    """Add what is pending; the next sublayer's row sum_s inp[s] x_s into ``u`` [T, W] fp32, its 1 / rms into ``rstd``."""
    if not u.is_cuda:
        u.copy_(xs.read(inp))
        rstd.copy_(1.0 / torch.sqrt((u * u).mean(-1) + eps))
        return
    xs._launch(0, 1, u.shape[0], None, inp, None, eps, u, rstd, None, None, None, None, True)


def norm(xs: Streams, inp, w, eps: float, h) -> torch.Tensor:
    """Add what is pending; the next sublayer's row, normed, into ``h`` [T, W]."""
    if not h.is_cuda:
        return h.copy_(ref.rms_rows(xs.read(inp), eps) * w)
    xs._launch(1, _act(h.dtype), h.shape[0], None, inp, w, eps, None, None, None, None, None, h, True)
    return h


def last_norm(xs: Streams, w, eps: float, dtype, rows=None) -> torch.Tensor:
    """The normed sum of the streams (``rows``: int32 indices, else all); the streams themselves are not stored."""
    n = xs.e.shape[0] if rows is None else rows.numel()
    if not xs.e.is_cuda:
        h = ref.rms_rows(xs.read(None), eps) * w
        return (h if rows is None else h[rows.long()]).to(dtype)
    if rows is not None:
        _req(rows, torch.int32, "rows")
    out = torch.empty(n, xs.e.shape[1], dtype=dtype, device=xs.e.device)
    xs._launch(1, _act(dtype), n, rows, None, w, eps, None, None, None, None, None, out, False)
    return out


def conv_decode(xs: Streams, inp, w, eps: float, conv, positions, tail: Tail, h) -> torch.Tensor:
    """One token per sequence: as :func:`norm`, the normed row then as h + conv(h) (``conv`` [taps, W]) with its earlier
    inputs in the sequences' slots (``tail``)."""
    if not h.is_cuda:
        n = ref.rms_rows(xs.read(inp), eps) * w
        por = [(b, 1, int(positions[b]), b) for b in range(n.shape[0])]
        return h.copy_(ref.input_conv(n, por, tail.block_tables, tail.rows, [conv])[0])
    _req(positions, torch.int32, "positions")
    xs._launch(2, _act(h.dtype), h.shape[0], None, inp, w, eps, None, None, conv, positions, tail, h, True)
    return h
