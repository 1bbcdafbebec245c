"""Residual branches between two RMS norms (csrc/kernels/branch.hip): 32-bit stream in place, the next sublayer's input
out of the same pass.

GPU tensors go to the native library (which must be built), CPU tensors to the fp32 reference.
"""
from __future__ import annotations

import dataclasses

import torch

from . import reference as ref
from ._native import check, kernels
from .kernels import _p, _req, _stream
from .stream import _act


@dataclasses.dataclass
class Branch:
    """A sublayer's result y on its way into the stream: x += y / rms(y) gain, with y one of
      ``y``                fp32 slabs [split, T, W] of a product
      ``y``, ``y2``        two products' slabs: factor (y / rms(y) w + y2 / rms(y2) w2)
      ``routed``           (rows [M, W] activations, row, weight and choice per (token, choice), experts, the sublayer's
                           input [T, W]): choices >= experts count the input itself
    ``gain`` fp32 [1] (all channels) or [W]."""
    gain: torch.Tensor
    eps: float
    y: torch.Tensor | None = None
    w: torch.Tensor | None = None
    y2: torch.Tensor | None = None
    w2: torch.Tensor | None = None
    factor: float = 0.5
    routed: tuple | None = None

    def value(self) -> torch.Tensor:
        """CPU: y."""
        if self.w is not None:
            return self.factor * (ref.rms_rows(self.y.sum(0), self.eps) * self.w + ref.rms_rows(self.y2.sum(0), self.eps) * self.w2)
        y = self.y.sum(0) if self.y is not None else 0.0
        if self.routed is not None:
            rows, pos, wt, ids, n, own = self.routed
            r = torch.where((ids >= n)[..., None], own.float()[:, None], rows[pos.long()].float())
            y = y + (r * wt[..., None]).sum(1)
        return y


def _vec(g, W) -> int:
    if g.numel() not in (1, W):
        raise ValueError(f"branch_norm: gain of {g.numel()} for rows of {W}")
    return int(g.numel() == W and W > 1)


def branch_norm(x: torch.Tensor, b: Branch | None, next_gain: torch.Tensor | None, eps: float, h: torch.Tensor | None) -> None:
    """Add the branch (if any) to ``x`` [T, W] in place; then x / rms(x) next_gain into ``h`` (if any)."""
    T, W = x.shape
    if not x.is_cuda:
        if b is not None:
            x.add_(ref.rms_rows(b.value(), b.eps) * b.gain)
        if h is not None:
            h.copy_(ref.rms_rows(x, eps) * next_gain)
        return
    _req(x, torch.float32, "x")
    dt = torch.float32 if h is None else h.dtype
    args = [None, 0, None, None, 0, None, 0.0] + [None] * 4 + [0, 0, None, None, 0]
    if b is not None:
        for name, p in (("y", b.y), ("y2", b.y2)):
            if p is not None:
                _req(p, torch.float32, name)
                if p.shape[1:] != (T, W):
                    raise ValueError(f"branch_norm: {name} {tuple(p.shape)} for a stream of {T} x {W}")
        rows = pos = wt = ids = own = None
        n = 0
        if b.routed is not None:
            rows, pos, wt, ids, n, own = b.routed
            dt = rows.dtype
            _req(own, dt, "own input")
            for name, t, d in (("row per choice", pos, torch.int32), ("choice", ids, torch.int32), ("weight", wt, torch.float32)):
                _req(t, d, name)
            if own.shape != (T, W) or ids.shape != pos.shape or wt.shape != pos.shape or rows.shape[1] != W or not rows.is_contiguous():
                raise ValueError(f"branch_norm: routed rows {tuple(rows.shape)}, choices {tuple(ids.shape)}")
        if h is not None and h.dtype != dt:
            raise TypeError(f"branch_norm: rows in {dt}, output in {h.dtype}")
        args = [_p(b.y), b.y.shape[0] if b.y is not None else 0, _p(b.w), _p(b.y2), b.y2.shape[0] if b.y2 is not None else 0, _p(b.w2),
                float(b.factor), _p(rows), _p(pos), _p(wt), _p(ids), ids.shape[1] if ids is not None else 0, n, _p(own),
                b.gain.data_ptr(), _vec(b.gain, W)]
    if h is not None and (h.shape != x.shape or not h.is_contiguous()):
        raise ValueError(f"branch_norm: h {tuple(h.shape)} for a stream of {T} x {W}")
    check(kernels().cfc_branch_norm(_act(dt), int(b is not None), *args, float(eps), x.data_ptr(), T, W, _p(next_gain),
                                    _vec(next_gain, W) if next_gain is not None else 0, _p(h), _stream(x)), "cfc_branch_norm")
