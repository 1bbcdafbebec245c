"""Routed experts (csrc/kernels/moe.hip and the grouped forms of dgemm.hip / pgemm.hip).

GPU tensors go to the native library (which must be built), CPU tensors to the fp32 reference.
"""
from __future__ import annotations

import dataclasses
import math

import torch

from . import kernels as K
from . import reference as ref
from ._native import check, kernels
from .cols import Cols
from .kernels import _p, _req, _stream
from .stream import _act, clamped_glu

GEMV_PAIRS = 8          # at most so many (token, choice) pairs each stream their own expert
ANY_TILE = 32           # rows per tile of the general products
MAX_EXPERTS = 1024
INF = float("inf")


@dataclasses.dataclass
class Router:
    experts: int
    top: int
    groups: int
    keep: int
    scale: float
    correction: torch.Tensor      # [experts] fp32
    softmax: bool = False         # scores: softmax over all outputs, else sigmoid
    renorm: bool = True           # weights over their sum


@dataclasses.dataclass(frozen=True)
class Glu:
    """Constants of an expert's gated activation: g = min(gate, limit), g sigmoid(alpha g) (clamp(up, +-limit) + beta)."""
    limit: float = INF
    alpha: float = 1.0
    beta: float = 0.0

    def args(self):
        return [float(self.limit), float(self.alpha), float(self.beta)]


class ExpertWeights:
    """Gate, up and down matrices of all experts.  Packed for the MFMA products where the width fits (``packed``;
    the inner size is padded to a multiple of 64 with zeros), row-major otherwise."""

    def __init__(self, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor):
        """gate, up [E, F, W], down [E, W, F]."""
        E, F, W = gate.shape
        self.E, self.F, self.W, self.dtype = E, F, W, gate.dtype
        self.packed = gate.is_cuda and gate.dtype == torch.bfloat16 and W % 64 == 0
        self.pair_order = None if not self.packed else torch.arange(GEMV_PAIRS, dtype=torch.int32, device=gate.device)
        if not self.packed:
            self.gu = torch.cat([gate, up], 1).contiguous()
            self.down = down.contiguous()
            return
        FP = 64 * math.ceil(F / 64)
        self.F = FP
        # wide tiles: 7 - 13 % faster than 64 rows once a batch reaches all experts
        self.bn_gu = 128 if (2 * FP) % 128 == 0 else 64
        self.bn_down = 128 if W % 128 == 0 else 64
        self.gu = torch.empty(E, 2 * FP * W, dtype=gate.dtype, device=gate.device)
        self.down = torch.empty(E, W * FP, dtype=gate.dtype, device=gate.device)
        for e in range(E):
            gu = torch.zeros(2 * FP, W, dtype=gate.dtype, device=gate.device)
            gu[:F], gu[FP:FP + F] = gate[e], up[e]
            self.gu[e] = K.pack_dgemm_weight(ref.interleave_gate_up(gu), bn=self.bn_gu).data
            d = torch.zeros(W, FP, dtype=gate.dtype, device=gate.device)
            d[:, :F] = down[e]
            self.down[e] = K.pack_dgemm_weight(d, bn=self.bn_down).data

    def nbytes(self) -> int:
        return (self.gu.numel() + self.down.numel()) * self.gu.element_size()

    def tile(self, pairs: int) -> int:
        """Rows per tile for this many (token, choice) pairs: whole 256-row tiles once the experts fill them."""
        if not self.packed:
            return ANY_TILE
        per = pairs / self.E
        return 64 if per <= 96 else 128 if per <= 160 else 256


def route(logits: Cols, r: Router) -> tuple[torch.Tensor, torch.Tensor]:
    """(expert per (token, choice) int32, weight fp32) of the router logits' fp32 slabs."""
    if not logits.t.is_cuda:
        return ref.route(logits.value(), r.correction, r.groups, r.keep, r.top, r.scale, r.softmax, r.renorm)
    if not logits.slabs:
        raise ValueError("route: fp32 slabs needed")
    T = logits.rows
    ids = torch.empty(T, r.top, dtype=torch.int32, device=logits.t.device)
    w = torch.empty(T, r.top, dtype=torch.float32, device=logits.t.device)
    p, split, ld, plane = logits.args()
    check(kernels().cfc_moe_route(p, split, ld, plane, r.correction.data_ptr(), T, r.experts, r.groups, r.keep, r.top,
                                  float(r.scale), int(r.softmax), int(r.renorm), ids.data_ptr(), w.data_ptr(), _stream(ids)),
          "cfc_moe_route")
    return ids, w


def sort_rows(ids, experts: int, tile: int):
    """(token per row, row per pair [T, top], expert per tile) of ops.reference.moe_rows, on ids' device."""
    T, top = ids.shape
    if not ids.is_cuda:
        return tuple(torch.from_numpy(a) for a in ref.moe_rows(ids, experts, tile))
    _req(ids, torch.int32, "ids")
    n = ref.moe_max_tiles(T * top, experts, tile)
    rows = torch.empty(n * tile, dtype=torch.int32, device=ids.device)
    pos = torch.empty(T, top, dtype=torch.int32, device=ids.device)
    te = torch.empty(n, dtype=torch.int32, device=ids.device)
    check(kernels().cfc_moe_rows(ids.data_ptr(), T * top, top, experts, tile, n, rows.data_ptr(), pos.data_ptr(), te.data_ptr(),
                                 _stream(ids)), "cfc_moe_rows")
    return rows, pos, te


def _grouped(glu: Glu | None, x, w, E, N, bn, tile, rows, te, out):
    """One grouped product over packed weights, gated with ``glu``."""
    M, Kd, lib = te.numel() * tile, x.shape[1], kernels()
    if not x.is_contiguous() or out.shape[0] != M:
        raise ValueError(f"grouped product: x {tuple(x.shape)}, out {tuple(out.shape)} for {M} rows")
    on, consts = int(glu is not None), (glu or Glu()).args()
    if tile == 256:
        check(lib.cfc_pgemm_group(on, x.data_ptr(), x.shape[0], w.data_ptr(), M, N, Kd, bn // 16, _p(rows), te.data_ptr(),
                                  out.data_ptr(), out.stride(0), *consts, _stream(x)), "cfc_pgemm_group")
    else:
        check(lib.cfc_dgemm_group(on, x.data_ptr(), w.data_ptr(), M, N, Kd, bn, tile, _p(rows), te.data_ptr(), out.data_ptr(),
                                  out.stride(0), *consts, _stream(x)), "cfc_dgemm_group")


def _experts_gemv(x, w: ExpertWeights, ids, glu: Glu) -> tuple[torch.Tensor, torch.Tensor]:
    """Few pairs: each streams its expert's matrices, in the pairs' own order."""
    T, top = ids.shape
    pairs, lib, dev = T * top, kernels(), x.device
    split, waves = K.gemv_packed_config(pairs * 2 * w.F, w.W, w.bn_gu // 16)
    part = K._workspace(dev, split * pairs * 2 * w.F)[:split * pairs * 2 * w.F].view(split, pairs, 2 * w.F)
    check(lib.cfc_gemv_group(x.data_ptr(), w.gu.data_ptr(), ids.data_ptr(), pairs, top, w.E, 2 * w.F, w.W, w.bn_gu // 16, 0,
                             part.data_ptr(), None, split, waves, _stream(x)), "cfc_gemv_group")
    a = clamped_glu(part, torch.empty(pairs, w.F, dtype=x.dtype, device=dev), *glu.args(), interleaved=True)
    y = torch.empty(pairs, w.W, dtype=x.dtype, device=dev)
    _, waves = K.gemv_packed_config(pairs * w.W, w.F, w.bn_down // 16, slab=False)
    check(lib.cfc_gemv_group(a.data_ptr(), w.down.data_ptr(), ids.data_ptr(), pairs, 1, w.E, w.W, w.F, w.bn_down // 16, 1, None,
                             y.data_ptr(), 1, waves, _stream(x)), "cfc_gemv_group")
    return y, w.pair_order[:pairs].view(T, top)


def experts(x, w: ExpertWeights, ids, glu: Glu = Glu()) -> tuple[torch.Tensor, torch.Tensor]:
    """W_down glu(W_gate x, W_up x) of every (token, choice): (rows [M, W] in x's dtype, row per pair [T, top]).  Choices
    past the last expert have no row of their own: what their place holds does not count."""
    if w.packed and ids.numel() <= GEMV_PAIRS and x.is_contiguous():
        _req(x, torch.bfloat16, "x")
        _req(ids, torch.int32, "ids")
        return _experts_gemv(x, w, ids, glu)
    tile = w.tile(ids.numel())
    rows, pos, te = sort_rows(ids, w.E, tile)
    M = te.numel() * tile
    y = torch.empty(M, w.W, dtype=x.dtype, device=x.device)
    if not x.is_cuda:
        y.zero_()
        for i, e in enumerate(te.tolist()):
            if e < 0:
                continue
            s = slice(i * tile, (i + 1) * tile)
            gu = x[rows[s].long()].float() @ w.gu[e].float().t()
            g, u = gu.chunk(2, -1)
            a = ref.clamped_glu(g, u, *glu.args()).to(x.dtype)
            y[s] = (a.float() @ w.down[e].float().t()).to(x.dtype)
        return y, pos
    a = torch.empty(M, w.F, dtype=x.dtype, device=x.device)
    if w.packed:
        _grouped(glu, x, w.gu, w.E, 2 * w.F, w.bn_gu, tile, rows, te, a)
        _grouped(None, a, w.down, w.E, w.W, w.bn_down, tile, None, te, y)
        return y, pos
    lib, f32 = kernels(), _act(x.dtype)
    if x.dtype != w.dtype or not x.is_contiguous():
        raise ValueError(f"experts: activations {x.dtype}, weights {w.dtype}")
    check(lib.cfc_moe_any(f32, 1, x.data_ptr(), w.gu.data_ptr(), M, w.F, w.W, rows.data_ptr(), te.data_ptr(), tile, a.data_ptr(),
                          w.F, *glu.args(), _stream(x)), "cfc_moe_any")
    check(lib.cfc_moe_any(f32, 0, a.data_ptr(), w.down.data_ptr(), M, w.W, w.F, None, te.data_ptr(), tile, y.data_ptr(), w.W,
                          *Glu().args(), _stream(x)), "cfc_moe_any")
    return y, pos
