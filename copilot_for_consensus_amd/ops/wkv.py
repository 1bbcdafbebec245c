"""Linear recurrence with data-dependent per-channel decay (csrc/kernels/wkv.hip).

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
from .kernels import _p, _req, _stream
from .stream import _act

CHUNK = 16               # tokens per chunk of the prompt kernels
MAX_CHUNKED_DIM = 128    # head sizes they are built for
MAX_DIM = 512


@dataclasses.dataclass
class Wkv:
    """A mixer's parameters: ``w2`` [H D, R] (bf16), ``w0``, ``norm`` [H D], ``u`` [H, D] fp32."""
    H: int
    D: int
    R: int
    w2: torch.Tensor
    w0: torch.Tensor
    u: torch.Tensor
    norm: torch.Tensor
    eps: float

    def __post_init__(self):
        if self.D > MAX_DIM or (self.D % 4 and self.D > 256):
            raise ValueError(f"recurrence head size {self.D} not supported (at most {MAX_DIM})")
        RP = 32 * math.ceil(self.R / 32)
        w2 = torch.zeros(self.H * self.D, RP, dtype=torch.bfloat16, device=self.w2.device)
        w2[:, :self.R] = self.w2
        self.w2 = w2

    def tail(self):
        return [self.w2.data_ptr(), self.w0.data_ptr(), self.u.data_ptr(), self.norm.data_ptr(), float(self.eps), self.H, self.D]


def chunk_plan(cu) -> tuple[np.ndarray, np.ndarray]:
    """(chunks [n, 2]: first row and rows, first chunk per portion [portions + 1]) of packed portions."""
    chunks, at = [], [0]
    for a, b in zip(cu, cu[1:]):
        chunks += [(r, min(CHUNK, b - r)) for r in range(a, b, CHUNK)]
        at.append(len(chunks))
    return np.asarray(chunks, np.int32), np.asarray(at, np.int32)


def _ref(p: Wkv, r, k, v, g, w1, slots, cu, ctx, state, out):
    T = out.shape[0]

    def heads(c):
        return c.value().view(T, p.H, p.D)
    w = ref.wkv_decay(w1.value(), p.w2[:, :p.R], p.w0).view(T, p.H, p.D)
    R, K, V = heads(r), heads(k), heads(v)
    for s, slot in enumerate(slots.tolist()):
        a, b = int(cu[s]), int(cu[s + 1])
        if int(ctx[s]) == b - a:
            state[slot].zero_()
        o = ref.wkv(R[a:b], K[a:b], V[a:b], w[a:b], p.u, state[slot])
        out[a:b] = ref.wkv_out(o, p.norm, g.value()[a:b], p.eps).to(out.dtype)
    return out


def step(p: Wkv, r: Cols, k: Cols, v: Cols, g: Cols, w1: Cols, slots, ctx_lens, state, out, cu_q=None) -> torch.Tensor:
    """Token by token: one token per sequence, or portions (``cu_q``).  ``r``, ``k``, ``v``, ``g`` columns of one product
    layout; ``w1`` the low-rank pre-activations; state [slots, H, D, D] fp32, updated; ``out`` [T, H D]."""
    if not out.is_cuda:
        return _ref(p, r, k, v, g, w1, slots, torch.arange(len(slots) + 1) if cu_q is None else cu_q, ctx_lens, state, out)
    a = [c.args(out.dtype) for c in (r, k, v, g)]
    if any(x[1:] != a[0][1:] for x in a):
        raise ValueError("wkv step: r, k, v and g must share strides")
    _req(slots, torch.int32, "slots")
    _req(ctx_lens, torch.int32, "ctx_lens")
    check(kernels().cfc_wkv_step(_act(out.dtype), *(x[0] for x in a), *a[0][1:], *w1.args(out.dtype), p.R, p.w2.shape[1],
                                 *p.tail(), slots.numel(), slots.data_ptr(), _p(cu_q), ctx_lens.data_ptr(), state.data_ptr(),
                                 out.data_ptr(), out.stride(0), _stream(out)), "cfc_wkv_step")
    return out


def prefill(p: Wkv, r: Cols, k: Cols, v: Cols, g: Cols, w1: Cols, slots, cu_q, ctx_lens, chunks, chunk_cu, state, out):
    """Packed portions, in chunks of 16 tokens (``chunks``, ``chunk_cu`` of :func:`chunk_plan` on the device)."""
    if not out.is_cuda:
        return _ref(p, r, k, v, g, w1, slots, cu_q, ctx_lens, state, out)
    widest = max(out.stride(0), v.t.stride(-2), g.t.stride(-2)) * out.element_size()
    if p.D > MAX_CHUNKED_DIM or (chunks.shape[0] + 4) * CHUNK * widest >= 2 ** 31 - 256:
        return step(p, r, k, v, g, w1, slots, ctx_lens, state, out, cu_q)
    T, RP, lib = out.shape[0], p.w2.shape[1], kernels()
    a = [c.args(out.dtype) for c in (r, k, v, g)]
    if any(x[1] for x in a):
        raise ValueError("wkv prefill: r, k, v and g are activations")
    for name, t in (("slots", slots), ("cu_q", cu_q), ("ctx_lens", ctx_lens), ("chunks", chunks), ("chunk_cu", chunk_cu)):
        _req(t, torch.int32, name)
    th = torch.empty(T, 3, RP, dtype=torch.bfloat16, device=out.device)
    check(lib.cfc_wkv_tanh(_act(out.dtype), *w1.args(out.dtype), T, p.R, RP, th.data_ptr(), _stream(out)), "cfc_wkv_tanh")
    n = chunks.shape[0]
    rec = torch.empty(n * p.H * lib.cfc_wkv_chunk_floats(p.D), dtype=torch.float32, device=out.device)
    ops = [x for c in a for x in (c[0], c[2])]
    check(lib.cfc_wkv_chunked(_act(out.dtype), *ops, th.data_ptr(), RP, *p.tail(), n, slots.numel(), chunk_cu.data_ptr(),
                              chunks.data_ptr(), slots.data_ptr(), cu_q.data_ptr(), ctx_lens.data_ptr(), rec.data_ptr(),
                              state.data_ptr(), out.data_ptr(), out.stride(0), _stream(out)), "cfc_wkv_chunked")
    return out
