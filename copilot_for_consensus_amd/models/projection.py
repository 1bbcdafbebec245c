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
from ..ops.stream import clamped_glu


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

    def slabs(self, x: torch.Tensor) -> torch.Tensor:
        """fp32 k-slice slabs [split, M, N] whose sum is the product (unrounded).  They may live in the
        stream's split-K workspace: consume them before the next product."""
        k = self._kernel(x)
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

    def glu(self, x: torch.Tensor, out: torch.Tensor, limit: float, alpha: float, beta: float) -> torch.Tensor:
        """W = 8-row interleaved gate / up rows, packed: the clamped GLU of the product into ``out`` [M, N / 2]
        (row-strided), in the product's epilogue where one pass over W fills the chip."""
        k, M = self._kernel(x), x.shape[0]
        if k == "pgemm" and self.K >= 128 and out.stride(0) % 8 == 0 and out.data_ptr() % 16 == 0:
            return K.pgemm_glu(x, self.packed, out, limit, alpha, beta)
        if k in ("pgemm", "dgemm") and self.N // self.packed.bn * -(-M // 256) >= K.DGEMM_CUS // 2 \
                and out.stride(0) % 4 == 0 and out.data_ptr() % 8 == 0:
            return K.dgemm_glu(x, self.packed, out, limit, alpha, beta)
        return clamped_glu(self.slabs(x), out, limit, alpha, beta, interleaved=True)

    def f32(self, x: torch.Tensor) -> torch.Tensor:
        """[M, N] fp32, a tensor of its own."""
        k = self._kernel(x)
        if k == "gemv":
            return K.gemv(x, self.packed, "f32")
        if k == "dgemm":
            out = torch.empty(1, x.shape[0], self.N, dtype=torch.float32, device=x.device)
            return K.dgemm(x, self.packed, "part", 1, part=out)[0]
        return self.slabs(x)[0]
