"""Minimal gated recurrence (csrc/kernels/gru.hip): S_t = (1 - z) S_(t-1) + z c, gates from the current token alone.

GPU tensors go to the native library (which must be built), CPU tensors to the fp32 reference.
"""
from __future__ import annotations

import dataclasses

import numpy as np
import torch

from . import reference as ref
from ._native import check, kernels
from .cols import Cols
from .kernels import _req, _stream
from .stream import _act

CHUNK = 64               # tokens per chunk of the prompt kernels


@dataclasses.dataclass
class Gru:
    """Biases of the gate's and the candidate's pre-activations, fp32 [W]."""
    bz: torch.Tensor
    bx: torch.Tensor

    @property
    def width(self) -> int:
        return self.bz.numel()


def chunk_plan(cu, size: int = CHUNK) -> tuple[np.ndarray, np.ndarray]:
    """(chunks [n, 2]: first row and rows, first chunk per portion [portions + 1]) of packed portions."""
    chunks, at = [], [0]
    for a, b in zip(cu, cu[1:]):
        chunks += [(r, min(size, b - r)) for r in range(a, b, size)]
        at.append(len(chunks))
    return np.asarray(chunks, np.int32).reshape(-1, 2), np.asarray(at, np.int32)


def _ref(p: Gru, z, u, g, slots, cu, ctx, state, out, factor):
    Z, U, gate = z.value() + p.bz, u.value() + p.bx, g.value()
    for s, slot in enumerate(slots.tolist()):
        a, b = int(cu[s]), int(cu[s + 1])
        if int(ctx[s]) == b - a:
            state[slot].zero_()
        out[a:b] = (ref.min_gru(Z[a:b], U[a:b], state[slot]) * gate[a:b] * torch.sigmoid(gate[a:b]) * factor).to(out.dtype)
    return out


def _fits(p: Gru, cols, out, state):
    if any(c.n != p.width for c in cols) or out.shape[1] != p.width or out.stride(1) != 1 or state.shape[-1] != p.width:
        raise ValueError(f"gru: columns {[c.n for c in cols]}, out {tuple(out.shape)} for a width of {p.width}")
    return [c.args(out.dtype) for c in cols]


def step(p: Gru, z: Cols, u: Cols, g: Cols, slots, ctx_lens, state, out, factor: float = 1.0) -> torch.Tensor:
    """One token per sequence: factor S silu(g) into ``out`` [B, W] (row-strided); state [slots, W] fp32, updated."""
    if not out.is_cuda:
        return _ref(p, z, u, g, slots, torch.arange(len(slots) + 1), ctx_lens, state, out, factor)
    _req(slots, torch.int32, "slots")
    _req(ctx_lens, torch.int32, "ctx_lens")
    ops = [x for c in _fits(p, (z, u, g), out, state) for x in c]
    check(kernels().cfc_gru_step(_act(out.dtype), *ops, p.bz.data_ptr(), p.bx.data_ptr(), slots.data_ptr(), ctx_lens.data_ptr(), out.shape[0],
                                 p.width, state.data_ptr(), out.data_ptr(), out.stride(0), float(factor), _stream(out)), "cfc_gru_step")
    return out


def prefill(p: Gru, z: Cols, u: Cols, g: Cols, slots, cu_q, ctx_lens, chunks, chunk_cu, state, out, factor: float = 1.0) -> torch.Tensor:
    """Packed portions, ``z``, ``u``, ``g`` activations (``chunks``, ``chunk_cu`` of :func:`chunk_plan` on the device)."""
    if not out.is_cuda:
        return _ref(p, z, u, g, slots, cu_q, ctx_lens, state, out, factor)
    for name, t in (("slots", slots), ("cu_q", cu_q), ("ctx_lens", ctx_lens), ("chunks", chunks), ("chunk_cu", chunk_cu)):
        _req(t, torch.int32, name)
    ops = _fits(p, (z, u, g), out, state)
    if any(c[1] for c in ops):
        raise ValueError("gru prefill: z, u and g are activations")
    n = chunks.shape[0]
    sums = torch.empty(n * 2 * p.width, dtype=torch.float32, device=out.device)
    check(kernels().cfc_gru_prefill(_act(out.dtype), *(x for c in ops for x in (c[0], c[2])), p.bz.data_ptr(), p.bx.data_ptr(),
                                    chunks.data_ptr(), n, chunk_cu.data_ptr(), cu_q.data_ptr(), ctx_lens.data_ptr(), slots.data_ptr(), slots.numel(), p.width, sums.data_ptr(),
                                    state.data_ptr(), out.data_ptr(), out.stride(0), float(factor), _stream(out)), "cfc_gru_prefill")
    return out
