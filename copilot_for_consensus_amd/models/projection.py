"""One weight matrix and the products a model takes with it, on the kernel that fits the row count.

The selection is DecoderModel's: at most K.GEMV_MAX_M rows on the packed GEMV, prompt-sized batches on
the hand-written prefill GEMM, what lies between on the decode GEMM, all three reading one fragment-
packed bf16 copy.  Shapes those kernels do not take (N or K not a multiple of 64) and 32-bit weights use
the library product.  CPU tensors: torch.
"""
from __future__ import annotations

import os

import torch
import torch.nn.functional as F

from ..ops import kernels as K
from ..ops.cols import Cols
from ..ops.stream import clamped_glu, relu_sq


class Projection:
    """y = x W^T for W [N, K], sharded by the caller.  bf16 on the GPU: packed when the shape fits."""

    # swiglu: interleaved gate / up rows, tiled for a product without split (its epilogue gates)
    __slots__ = ("w", "packed", "N", "K", "min_tiles")

    def __init__(self, w: torch.Tensor, decode_rows: int = 128, swiglu: bool = False):
        self.N, self.K = w.shape
        self.packed = None
        self.w = w.contiguous()
        # fewer 256 x 256 output tiles than this run on the decode GEMM (DecoderModel.PGEMM_MIN_TILES)
        self.min_tiles = 96
        if self.packs(w, self.N, self.K):
            self.packed = K.pack_dgemm_weight(self.w, swiglu=swiglu, m=decode_rows)
            self.w = None

    @staticmethod
    def packs(w: torch.Tensor, N: int, K: int) -> bool:
        """Whether an [N, K] matrix like ``w`` is packed for the hand-written products."""
        return (w.is_cuda and w.dtype == torch.bfloat16 and N % 64 == 0 and K % 64 == 0
                and os.environ.get("CFC_DECODE_PACKED", "auto") != "0")

    def rowmajor(self) -> torch.Tensor:
        return self.w if self.w is not None else K._rowmajor(self.packed)

    def nbytes(self) -> int:
        return self.packed.nbytes() if self.packed is not None else self.w.numel() * self.w.element_size()

    @classmethod
    def of_packed(cls, packed: "K.PackedWeight"):
        """A projection over (a run of tiles of) a packed matrix."""
        p = cls.__new__(cls)
        p.N, p.K, p.w, p.packed, p.min_tiles = packed.N, packed.K, None, packed, 96
        return p

    def _prefill(self, M: int) -> bool:
        return M >= 256 and -(-M // 256) * -(-self.N // 256) >= self.min_tiles and M * self.K * 2 < 2 ** 32

    def _kernel(self, x) -> str:
        if self.packed is None or not x.is_contiguous():
            return "lib"
        if x.shape[0] <= K.GEMV_MAX_M:
            return "gemv"
        return "pgemm" if self._prefill(x.shape[0]) else "dgemm"

    def act(self, x: torch.Tensor) -> torch.Tensor:
        """[M, N] in x's dtype."""
        k = self._kernel(x)
        if k == "lib":
            return F.linear(x, self.rowmajor())
        if k == "gemv":
            return K.splitk_reduce(K.gemv_part(x, self.packed))
        if k == "pgemm":
            return K.pgemm(x, self.packed, "bf16", variant="ppp")
        return K.dgemm_linear(x, self.packed)

    def slabs(self, x: torch.Tensor, own: bool = False) -> torch.Tensor:
        """fp32 k-slice slabs [split, M, N] whose sum is the product (unrounded).  They may live in the
        stream's split-K workspace: consume them before the next product, unless they are to be a tensor of
        their ``own``."""
        k = self._kernel(x)
        if own and k in ("gemv", "dgemm"):
            M = x.shape[0]
            split = K.gemv_packed_config(self.N, self.K, self.packed.bn // 16, M)[0] if k == "gemv" else \
                K.dgemm_config(M, self.N, self.K, bn=self.packed.bn)[1]
            out = torch.empty(split, M, self.N, dtype=torch.float32, device=x.device)
            return K.gemv_part(x, self.packed, split, out=out) if k == "gemv" else \
                K.dgemm(x, self.packed, "part", split, part=out)
        if k == "gemv":
            return K.gemv_part(x, self.packed)
        if k == "pgemm":
            return K.pgemm(x, self.packed, "f32", variant="ppp")[None]
        if k == "dgemm":
            bn, split = K.dgemm_config(x.shape[0], self.N, self.K, bn=self.packed.bn)
            return K.dgemm(x, self.packed, "part", split, bn=bn)
        w = self.rowmajor()
        if x.is_cuda and x.dtype == torch.bfloat16:
            return torch.mm(x, w.t(), out_dtype=torch.float32)[None]
        return F.linear(x.float(), w.float())[None]

    def glu(self, x: torch.Tensor, out: torch.Tensor, limit: float, alpha: float, beta: float, cubic: float = 0.0) -> torch.Tensor:
        """W = 8-row interleaved gate / up rows: the clamped GLU of the product into ``out`` [M, N / 2]
        (row-strided), in the product's epilogue where one pass over (packed) W fills the chip."""
        k, M = self._kernel(x), x.shape[0]
        if k == "pgemm" and self.K >= 128 and out.stride(0) % 8 == 0 and out.data_ptr() % 16 == 0:
            return K.pgemm_glu(x, self.packed, out, limit, alpha, beta, cubic)
        if k in ("pgemm", "dgemm") and self.N // self.packed.bn * -(-M // 256) > K.DGEMM_CUS // 2 \
                and out.stride(0) % 4 == 0 and out.data_ptr() % 8 == 0:
            return K.dgemm_glu(x, self.packed, out, limit, alpha, beta, cubic)
        return clamped_glu(self.slabs(x), out, limit, alpha, beta, interleaved=True, cubic=cubic)

    def relu_sq(self, x: torch.Tensor) -> torch.Tensor:
        """relu(product)^2 [M, N] in x's dtype, in the prompt product's epilogue, else with the sum of the slabs."""
        k = self._kernel(x)
        if k == "pgemm" and self.K >= 128:
            return K.pgemm(x, self.packed, "relu2", variant="ppp")
        return relu_sq(self.slabs(x), x.dtype)

    def f32(self, x: torch.Tensor) -> torch.Tensor:
        """[M, N] fp32, a tensor of its own."""
        k = self._kernel(x)
        if k == "gemv":
            return K.gemv(x, self.packed, "f32")
        if k == "dgemm":
            out = torch.empty(1, x.shape[0], self.N, dtype=torch.float32, device=x.device)
            return K.dgemm(x, self.packed, "part", 1, part=out)[0]
        return self.slabs(x)[0]


class JointProjection:
    """Several matrices of one width read by one layer, each multiplying one of a few inputs [inputs, T, K]: one
    packed matrix (every part padded with zero rows to whole tiles).  A decode step runs them all in one launch; a
    prompt's rows take each part on its own."""

    def __init__(self, parts: list[tuple[torch.Tensor, int]]):
        """parts: (W [N, K], index of its input)."""
        self.sizes = [w.shape[0] for w, _ in parts]
        self.inputs = [i for _, i in parts]
        self.K = parts[0][0].shape[1]
        w0 = parts[0][0]
        self.packed = None
        pad, bn = (lambda n: n), 64
        if Projection.packs(w0, 64, self.K):
            total = {b: sum(-(-n // b) * b for n in self.sizes) for b in (64, 128)}
            bn = 128 if total[128] <= 1.03 * total[64] else 64
            pad = (lambda n: -(-n // bn) * bn)
        self.offsets, at = [], 0
        for n in self.sizes:
            self.offsets.append(at)
            at += pad(n)
        self.N = at
        if not Projection.packs(w0, 64, self.K):
            self.parts = [Projection(w) for w, _ in parts]
            return
        full = w0.new_zeros(at, self.K)
        for (w, _), o in zip(parts, self.offsets):
            full[o:o + w.shape[0]] = w
        self.packed = K.pack_dgemm_weight(full, bn=bn)
        ends = self.offsets[1:] + [at]
        self.parts = [Projection.of_packed(K.PackedWeight(self.packed.data[o * self.K:e * self.K], e - o, self.K, bn))
                      for o, e in zip(self.offsets, ends)]
        self.in_of = torch.tensor([i for i, o, e in zip(self.inputs, self.offsets, ends) for _ in range((e - o) // bn)],
                                  dtype=torch.int32, device=w0.device)

    def nbytes(self) -> int:
        return self.packed.nbytes() if self.packed is not None else sum(p.nbytes() for p in self.parts)

    def act(self, j: int, acts: torch.Tensor) -> Cols:
        """Part j's columns as activations."""
        return Cols(self.parts[j].act(acts[self.inputs[j]]), 0, self.sizes[j])

    def slabs(self, j: int, acts: torch.Tensor) -> Cols:
        """Part j's columns in fp32 (a tensor of its own)."""
        return Cols(self.parts[j].slabs(acts[self.inputs[j]], own=True), 0, self.sizes[j])

    def joint(self, acts: torch.Tensor) -> list[Cols]:
        """Every part's columns in fp32, of one product (a tensor of its own)."""
        M = acts.shape[1]
        if self.packed is None or not acts.is_contiguous():
            x = [F.linear(acts[i].float(), p.rowmajor().float()) for p, i in zip(self.parts, self.inputs)]
            out = torch.cat(x, 1)[None]            # no padding: the parts lie side by side
        else:
            gemv = M <= K.GEMV_MAX_M
            split = K.gemv_packed_config(self.N, self.K, self.packed.bn // 16, M)[0] if gemv else \
                K.dgemm_config(M, self.N, self.K, bn=self.packed.bn)[1]
            out = torch.empty(split, M, self.N, dtype=torch.float32, device=acts.device)
            if gemv:
                K.gemv_part(acts, self.packed, split, out=out, in_of=self.in_of)
            else:
                K.dgemm_joint(acts, self.packed, self.in_of, out)
        return [Cols(out, o, n) for o, n in zip(self.offsets, self.sizes)]
