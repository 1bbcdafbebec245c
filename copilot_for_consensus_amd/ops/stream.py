"""32-bit residual stream ops (csrc/kernels/stream.hip): depth average with its RMS norm, causal input
convolution with a paged tail, clamped GLU, logit softcap.

As in :mod:`.kernels`, GPU tensors go to the native library (which must be built) and CPU tensors to the
fp32 reference.  Activation outputs are bf16 or fp32, by the ``dtype`` / output tensor given.
"""
from __future__ import annotations

import numpy as np
import torch

from . import reference as ref
from ._native import check, kernels
from .kernels import _p, _req, _stream

KV_BLOCK = ref.KV_BLOCK


def _act(dtype) -> int:
    if dtype not in (torch.bfloat16, torch.float32):
        raise TypeError(f"activation dtype {dtype}: bfloat16 or float32")
    return int(dtype == torch.float32)


def sinusoid_turns(width: int, base: float, device) -> torch.Tensor:
    """Turns per position of the sinusoids of entries 2i and 2i + 1: base^(-2i / width) / 2 pi, in 64 bits."""
    i = np.arange((width + 1) // 2, dtype=np.float64)
    return torch.tensor(base ** (-2.0 * i / width) / (2.0 * np.pi), dtype=torch.float64, device=device)


def embed_f32(table: torch.Tensor, ids: torch.Tensor, out: torch.Tensor, scale: float = 1.0, positions=None, turns=None) -> torch.Tensor:
    """Token rows times ``scale`` as fp32 into ``out`` [T, W]; with ``positions`` plus their sinusoids (``turns`` of
    :func:`sinusoid_turns`)."""
    if not table.is_cuda:
        out.copy_(table[ids.long()])
        if scale != 1.0:
            out.mul_(scale)
        if positions is not None:
            out.add_(ref.sinusoids(positions, turns, out.shape[1]))
        return out
    _req(ids, torch.int32, "ids")
    _req(out, torch.float32, "out")
    if positions is not None:
        _req(positions, torch.int32, "positions")
        _req(turns, torch.float64, "turns")
    check(kernels().cfc_embed_f32(out.data_ptr(), table.data_ptr(), ids.data_ptr(), ids.numel(), table.shape[1],
                                  table.shape[0], _act(table.dtype), float(scale), _p(positions), _p(turns), _stream(table)),
          "cfc_embed_f32")
    return out


class Tail:
    """The input convolution's tail of one layer: rows [blocks, slots, W] fp32, paged, addressed by the batch's block
    tables; or (``block_tables`` one-dimensional) [sequence slots, ring, W], addressed by the batch's state slots."""

    __slots__ = ("rows", "block_tables")

    def __init__(self, rows, block_tables):
        self.rows, self.block_tables = rows, block_tables

    def args(self):
        if self.rows is None:
            return [None, 0, None, 1]
        _req(self.block_tables, torch.int32, "block tables or slots")
        paged = self.block_tables.dim() == 2
        return [self.rows.data_ptr(), self.rows.shape[1], self.block_tables.data_ptr(), self.block_tables.shape[1] if paged else 0]


class Update:
    """What a layer adds to the stream: fp32 slabs [split, T, W] of its sublayers' sum, an optional bias
    and the depth weights over X_0 .. X_n (n results so far, the new one becomes X_n).  ``pre`` [T, W]: the
    first ``j0`` terms of the average, already summed (:func:`depth_pre`)."""

    __slots__ = ("part", "bias", "dwa", "n", "pre", "j0")

    def __init__(self, part, bias, dwa, n, pre=None, j0=0):
        self.part, self.bias, self.dwa, self.n, self.pre, self.j0 = part, bias, dwa, n, pre, j0

    def terms(self, x, hist, eps):
        """CPU: the averaged stream and its 1 / rms."""
        return ref.depth_norm(x, hist, self.part, self.bias, self.dwa, self.n, eps, self.pre, self.j0)


DEPTH_RUN = 4       # layers per depth_pre pass


def depth_pre(hist, n: int, dwas) -> torch.Tensor:
    """[len(dwas), T, W]: sum over j < n of dwa[j] X_j for each of (up to four) weight vectors."""
    pre = torch.empty(len(dwas), *hist.shape[1:], dtype=torch.float32, device=hist.device)
    if not hist.is_cuda:
        for p, w in zip(pre, dwas):
            p.copy_(torch.einsum("j,jtw->tw", w[:n].float(), hist[:n]))
        return pre
    if len(dwas) > DEPTH_RUN or any(w.numel() < n for w in dwas) or hist.shape[0] < n:
        raise ValueError(f"depth_pre: {len(dwas)} weight vectors over {n} of {hist.shape[0]} results")
    ptrs = [w.data_ptr() for w in dwas] + [None] * (DEPTH_RUN - len(dwas))
    check(kernels().cfc_depth_pre(hist.data_ptr(), hist[0].numel(), n, len(dwas), *ptrs, pre.data_ptr(), _stream(hist)),
          "cfc_depth_pre")
    return pre


def _stats_ref(x, hist, up, eps):
    return up.terms(x, hist, eps) if up else ref.depth_norm(x, hist, None, None, None, 0, eps)


def _depth(mode, f32, nrows, rows, x, hist, up, norm_w, eps, x_out, rstd, h1, h2, w1, w2, positions, tail, ref_t):
    T, W = hist.shape[1], hist.shape[2]
    for name, t in (("x", x), ("hist", hist)):
        _req(t, torch.float32, name)
    if up is not None:
        _req(up.part, torch.float32, "part")
        if up.part.shape[1:] != (T, W) or hist.shape[0] <= up.n or up.dwa.numel() != up.n + 1:
            raise ValueError(f"depth_norm: part {tuple(up.part.shape)}, hist {tuple(hist.shape)}, dwa {up.dwa.numel()}")
    t = tail.args() if tail is not None else [None, 0, None, 1]
    check(kernels().cfc_depth_norm(
        mode, f32, nrows, _p(rows), x.data_ptr(), hist.data_ptr(), _p(up.part) if up else None,
        up.part.shape[0] if up else 0, _p(up.bias) if up else None, _p(up.dwa) if up else None, up.n if up else 0,
        _p(up.pre) if up else None, up.j0 if up else 0, _p(norm_w), float(eps), _p(x_out), _p(rstd), T, W, _p(h1), h1.stride(0) if h1 is not None else 0, _p(h2),
        h2.stride(0) if h2 is not None else 0, _p(w1), _p(w2), w1.shape[0] if w1 is not None else 1, _p(positions), *t,
        _stream(ref_t)), "cfc_depth_norm")


def depth_stats(x, hist, up: Update | None, eps: float, x_out, rstd) -> None:
    """Apply ``up`` (if any) and leave the averaged stream in ``x_out`` and 1 / rms per row in ``rstd``."""
    if not hist.is_cuda:
        y, r = _stats_ref(x, hist, up, eps)
        x_out.copy_(y)
        rstd.copy_(r)
        return
    _depth(0, 1, hist.shape[1], None, x, hist, up, None, eps, x_out, rstd, None, None, None, None, None, None, hist)


def depth_norm(x, hist, up: Update | None, norm_w, eps: float, dtype, rows=None) -> torch.Tensor:
    """Apply ``up`` and return the normed rows (``rows``: int32 indices, else all) in ``dtype``; the
    stream itself is not stored (the model's last norm)."""
    n = rows.numel() if rows is not None else hist.shape[1]
    if not hist.is_cuda:
        y, r = _stats_ref(x, hist, up, eps)
        h = y * r[:, None] * norm_w
        return (h if rows is None else h[rows.long()]).to(dtype)
    out = torch.empty(n, hist.shape[2], dtype=dtype, device=hist.device)
    if rows is not None:
        _req(rows, torch.int32, "rows")
    _depth(1, _act(dtype), n, rows, x, hist, up, norm_w, eps, None, None, out, None, None, None, None, None, hist)
    return out


def depth_conv_decode(x, hist, up: Update | None, norm_w, eps: float, convs, positions, tail: Tail, x_out, outs) -> None:
    """One token per sequence: apply ``up``, norm, and run the row through each sublayer's input
    convolution (``convs``: one or two [taps, W]) with the cached tail; results into ``outs``."""
    if not hist.is_cuda:
        y, r = _stats_ref(x, hist, up, eps)
        x_out.copy_(y)
        h = y * r[:, None] * norm_w
        por = [(b, 1, int(positions[b]), b) for b in range(h.shape[0])]
        for o, v in zip(outs, ref.input_conv(h, por, tail.block_tables, tail.rows, convs)):
            o[:, :v.shape[1]] = v.to(o.dtype)
        return
    two = len(convs) > 1
    _depth(2, _act(outs[0].dtype), hist.shape[1], None, x, hist, up, norm_w, eps, x_out, None, outs[0],
           outs[1] if two else None, convs[0], convs[1] if two else None, positions, tail, hist)


def conv_tiles(portions, rows: int | None = None) -> np.ndarray:
    """[2, n, 4] int32 tiles of :func:`input_conv`: each portion (first row, rows, first position,
    sequence) cut at the cache blocks' borders, or (tails in slots) after every ``rows`` of its rows, at least
    taps - 1; then per tile the portion's rows before it and in all."""
    tiles, lead = [], []
    for row0, n, pos0, seq in portions:
        r = 0
        while r < n:
            m = min(n - r, rows or KV_BLOCK - (pos0 + r) % KV_BLOCK)
            tiles.append((row0 + r, m, pos0 + r, seq))
            lead.append((r, n, 0, 0))
            r += m
    return np.asarray([tiles, lead], np.int32).reshape(2, -1, 4)


def input_conv(x, rstd, norm_w, convs, tiles, tail: Tail, outs) -> None:
    """Packed portions: h = x * rstd * norm_w and h + conv(h) of every sublayer into ``outs`` (row-strided
    views); ``tiles`` from :func:`conv_tiles`, on the device."""
    if not x.is_cuda:
        h = x * rstd[:, None] * norm_w
        t = tiles.tolist()
        por = []
        for (row0, n, pos0, seq), (lead, *_) in zip(*t):
            if lead:
                por[-1][1] += n
            else:
                por.append([row0, n, pos0, seq])
        for o, v in zip(outs, ref.input_conv(h, por, tail.block_tables, tail.rows, convs)):
            o[:, :v.shape[1]] = v.to(o.dtype)
        return
    _req(tiles, torch.int32, "tiles")
    two = len(convs) > 1
    check(kernels().cfc_input_conv(_act(outs[0].dtype), tiles.shape[1], tiles.data_ptr(), x.data_ptr(), rstd.data_ptr(),
                                   norm_w.data_ptr(), convs[0].data_ptr(), _p(convs[1]) if two else None,
                                   convs[0].shape[0], *tail.args(), x.shape[1], outs[0].data_ptr(), outs[0].stride(0),
                                   _p(outs[1]) if two else None, outs[1].stride(0) if two else 0, _stream(x)),
          "cfc_input_conv")


def clamped_glu(gu, out, limit: float, alpha: float, beta: float, gate_bias=None, up_bias=None,
                interleaved: bool = False, cubic: float = 0.0) -> torch.Tensor:
    """g = min(gate, limit), u = clamp(up, +-limit): g sigmoid(alpha g (1 + cubic g^2)) (u + beta) into ``out`` [T, F]
    (row-strided).
    ``gu`` [T, 2F], or fp32 slabs [split, T, 2F] to be summed: gate | up halves or the 8-column interleaved
    groups of ops.reference.interleave_gate_up."""
    T, F2 = gu.shape[-2:]
    split = gu.shape[0] if gu.dim() == 3 else 1
    if not gu.is_cuda:
        gu = gu.float().sum(0) if gu.dim() == 3 else gu.float()
        if interleaved:
            v = gu.view(T, -1, 2, ref.GU_GROUP)
            g, u = v[:, :, 0].reshape(T, -1), v[:, :, 1].reshape(T, -1)
        else:
            g, u = gu[:, :F2 // 2], gu[:, F2 // 2:]
        g = g + (gate_bias if gate_bias is not None else 0.0)
        u = u + (up_bias if up_bias is not None else 0.0)
        out.copy_(ref.clamped_glu(g, u, limit, alpha, beta, cubic))
        return out
    if not gu.is_contiguous() or out.shape != (T, F2 // 2):
        raise ValueError(f"clamped_glu: gate / up {tuple(gu.shape)} (contiguous), out {tuple(out.shape)}")
    check(kernels().cfc_clamped_glu(_act(out.dtype), _act(gu.dtype), out.data_ptr(), out.stride(0), gu.data_ptr(), split,
                                    _p(gate_bias), _p(up_bias), T, F2 // 2, int(interleaved), float(limit), float(alpha),
                                    float(beta), float(cubic), _stream(gu)), "cfc_clamped_glu")
    return out


def softcap_(logits: torch.Tensor, cap: float) -> torch.Tensor:
    """cap * tanh(logits / cap) in place (fp32)."""
    if not logits.is_cuda:
        return logits.copy_(cap * torch.tanh(logits / cap))
    _req(logits, torch.float32, "logits")
    check(kernels().cfc_softcap(logits.data_ptr(), logits.numel(), float(cap), _stream(logits)), "cfc_softcap")
    return logits


def relu_sq(x: torch.Tensor, dtype) -> torch.Tensor:
    """relu(sum of fp32 slabs [split, T, F])^2 as activations [T, F]."""
    if not x.is_cuda:
        return ref.relu_sq(x.sum(0)).to(dtype)
    _req(x, torch.float32, "x")
    out = torch.empty(x.shape[1:], dtype=dtype, device=x.device)
    check(kernels().cfc_relu_sq(_act(dtype), out.data_ptr(), x.data_ptr(), x.shape[0], out.numel(), _stream(x)), "cfc_relu_sq")
    return out
