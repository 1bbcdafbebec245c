"""Columns of a product as an operand of the kernel that consumes it: activations [T, N], or fp32 k-slice slabs
[split, T, N] whose sum is the product (a decode step's, never reduced by a launch of their own)."""
from __future__ import annotations

import torch


class Cols:
    __slots__ = ("t", "c0", "n")

    def __init__(self, t: torch.Tensor, c0: int = 0, n: int | None = None):
        self.t, self.c0, self.n = t, c0, t.shape[-1] - c0 if n is None else n
        if t.stride(-1) != 1 or self.c0 + self.n > t.shape[-1] or (t.dim() == 3 and t.dtype != torch.float32):
            raise ValueError(f"columns {c0}..{self.c0 + self.n} of {tuple(t.shape)} {t.dtype}")

    @property
    def slabs(self) -> bool:
        return self.t.dim() == 3

    @property
    def split(self) -> int:
        return self.t.shape[0] if self.slabs else 0

    @property
    def rows(self) -> int:
        return self.t.shape[-2]

    def value(self) -> torch.Tensor:
        """fp32 [T, n] (CPU)."""
        t = self.t.sum(0) if self.slabs else self.t.float()
        return t[:, self.c0:self.c0 + self.n]

    def args(self, act_dtype=None) -> list:
        """pointer, split (0: activations), row stride, slab stride."""
        if act_dtype is not None and not self.slabs and self.t.dtype != act_dtype:
            raise TypeError(f"columns in {self.t.dtype}, {act_dtype} needed")
        return [self.t.data_ptr() + self.c0 * self.t.element_size(), self.split, self.t.stride(-2),
                self.t.stride(0) if self.slabs else 0]
