"""Gated, post-normed residual branches and the token shift (csrc/kernels/gated.hip): 32-bit stream in place,
the layers' input rows of a sequence's last two tokens as its state.

GPU tensors go to the native library (which must be built), CPU tensors to the fp32 reference.
"""
from __future__ import annotations

import dataclasses

import torch

from . import reference as ref
from ._native import check, kernels
from .cols import Cols
from .kernels import _p, _req, _stream
from .stream import _act


@dataclasses.dataclass
class Branch:
    """A sublayer's result on its way into the stream: x += LayerNorm((y + y2 + routed rows) * sigmoid(gate + bias)) w.
    ``y``, ``y2``: fp32 slabs [split, T, W]; ``routed``: (rows [M, W] activations, row per (token, choice), weight
    per (token, choice)); ``gate``: pre-sigmoid columns."""
    gate: Cols
    gate_bias: torch.Tensor
    norm_w: torch.Tensor
    eps: float
    y: torch.Tensor | None = None
    y2: torch.Tensor | None = None
    routed: tuple | None = None

    def delta(self) -> torch.Tensor:
        """CPU: what the branch adds."""
        y = sum(p.sum(0) for p in (self.y, self.y2) if p is not None)
        if self.routed is not None:
            rows, pos, wt = self.routed
            y = y + (rows[pos.long()].float() * wt[..., None]).sum(1)
        return ref.layernorm_rows(y * torch.sigmoid(self.gate.value() + self.gate_bias), self.norm_w, self.eps)


@dataclasses.dataclass
class Shift:
    """Token shift ahead of a mixer: ``shift`` [W]; ``mus`` [n, W] mixes of the shifted row (None: the row itself);
    ``prev`` [slots, 2, W] the sequences' last two input rows of the layer."""
    shift: torch.Tensor
    mus: torch.Tensor | None
    prev: torch.Tensor

    @property
    def outputs(self) -> int:
        return 1 if self.mus is None else self.mus.shape[0]

    def acts(self, T: int, dtype) -> torch.Tensor:
        """Buffer of the sublayer's inputs [1 + outputs, T, W]: the row, then the shifted row or its mixes."""
        return torch.empty(1 + self.outputs, T, self.shift.numel(), dtype=dtype, device=self.shift.device)

    def args(self):
        return [self.shift.data_ptr(), _p(self.mus), 0 if self.mus is None else self.mus.shape[0]]


def shift_mix(x, sh: Shift, meta, positions, acts) -> None:
    """Packed portions: the inputs of a layer's products into ``acts``; ``meta`` the row words of ops.reference.row_meta."""
    T, W = x.shape
    if not x.is_cuda:
        xp, xpp = ref.before_rows(x, meta, positions, sh.prev)
        acts[0].copy_(x)
        for o, v in zip(acts[1:], ref.shift_mix(x, xp, xpp, positions, sh.shift, sh.mus)):
            o.copy_(v)
        return
    _req(x, torch.float32, "x")
    _req(meta, torch.int32, "meta")
    _req(positions, torch.int32, "positions")
    if not acts.is_contiguous() or acts.shape != (1 + sh.outputs, T, W):
        raise ValueError(f"shift_mix: acts {tuple(acts.shape)} for {sh.outputs} outputs of {T} x {W}")
    check(kernels().cfc_shift_mix(_act(acts.dtype), x.data_ptr(), meta.data_ptr(), positions.data_ptr(), *sh.args(),
                                  sh.prev.data_ptr(), T, W, acts.data_ptr(), _stream(x)), "cfc_shift_mix")


def _gated(mode, x, b: Branch | None, h, prev, meta, positions, sh: Shift | None, slots, acts, dtype):
    T, W = x.shape
    _req(x, torch.float32, "x")
    bargs = [None, 0, None, 0, None, None, None, 0, None, 0, 0, 0, 0, None, None, 0.0]
    if b is not None:
        for name, p in (("y", b.y), ("y2", b.y2)):
            if p is not None:
                _req(p, torch.float32, name)
                if p.shape[1:] != (T, W):
                    raise ValueError(f"gated_norm: {name} {tuple(p.shape)} for a stream of {T} x {W}")
        rows = pos = wt = None
        if b.routed is not None:
            rows, pos, wt = b.routed
            _req(rows, dtype, "routed rows")
            _req(pos, torch.int32, "routed positions")
            _req(wt, torch.float32, "routed weights")
        g = b.gate.args(dtype)
        bargs = [_p(b.y), b.y.shape[0] if b.y is not None else 0, _p(b.y2), b.y2.shape[0] if b.y2 is not None else 0,
                 _p(rows), _p(pos), _p(wt), pos.shape[1] if pos is not None else 0, g[0], int(not b.gate.slabs), g[1], g[2],
                 g[3], b.gate_bias.data_ptr(), b.norm_w.data_ptr(), float(b.eps)]
    sargs = sh.args() if sh is not None else [None, None, 0]
    if acts is not None and (not acts.is_contiguous() or acts.shape != (1 + sh.outputs, T, W)):
        raise ValueError(f"gated_norm: acts {tuple(acts.shape)} for {sh.outputs} outputs of {T} x {W}")
    check(kernels().cfc_gated_norm(mode, _act(dtype), *bargs, x.data_ptr(), T, W, _p(h), _p(prev), _p(meta), _p(positions),
                                   *sargs, _p(slots), _p(acts), _stream(x)), "cfc_gated_norm")


def gated_norm(x, b: Branch, dtype, h=None, prev=None, meta=None, positions=None) -> None:
    """Packed portions: add the branch to ``x`` in place; the new row into ``h`` (the next product's input).  With
    ``prev``: first store the portions' last rows of x there (the layer's input rows, for what comes later)."""
    if not x.is_cuda:
        if prev is not None:
            for t, (m, p) in enumerate(zip(meta.tolist(), positions.tolist())):
                if m & ref.META_TAIL:
                    prev[m >> ref.META_SLOT, p % 2] = x[t]
        x.add_(b.delta())
        if h is not None:
            h.copy_(x)
        return
    _gated(0, x, b, h, prev, meta, positions, None, None, None, dtype)


def gated_shift(x, b: Branch | None, dtype, h=None, sh: Shift | None = None, positions=None, slots=None, acts=None) -> None:
    """One token per sequence: add the branch (if any) to ``x`` in place, the new row into ``h``; then (``acts``) the
    next layer's token shift from and into the sequences' state."""
    if not x.is_cuda:
        if b is not None:
            x.add_(b.delta())
            if h is not None:
                h.copy_(x)
        if acts is not None:
            meta = slots.to(torch.int32) << ref.META_SLOT
            xp, xpp = ref.before_rows(x, meta, positions, sh.prev)
            acts[0].copy_(x)
            for o, v in zip(acts[1:], ref.shift_mix(x, xp, xpp, positions, sh.shift, sh.mus)):
                o.copy_(v)
            for t, (s, p) in enumerate(zip(slots.tolist(), positions.tolist())):
                sh.prev[s, p % 2] = x[t]
        return
    if acts is not None:
        _req(positions, torch.int32, "positions")
        _req(slots, torch.int32, "slots")
    _gated(1, x, b, h, sh.prev if sh is not None else None, None, positions, sh, slots, acts, dtype)


def final_norm(x, w, eps: float, dtype, rows=None) -> torch.Tensor:
    """LayerNorm of the rows ``rows`` (int32; None: all) of the stream."""
    if not x.is_cuda:
        return ref.layernorm_rows(x if rows is None else x[rows.long()], w, eps).to(dtype)
    n = x.shape[0] if rows is None else rows.numel()
    if rows is not None:
        _req(rows, torch.int32, "rows")
    out = torch.empty(n, x.shape[1], dtype=dtype, device=x.device)
    check(kernels().cfc_final_norm(_act(dtype), x.data_ptr(), _p(rows), n, w.data_ptr(), float(eps), x.shape[1], out.data_ptr(),
                                   _stream(x)), "cfc_final_norm")
    return out
