"""Paged KV cache sized for one MI355X (288 GB HBM3E).

Layout per layer (see csrc/kernels/attention.hip for why):
  K: [num_blocks, kv_heads, 32, head_dim]        (row = key)
  V: [num_blocks, kv_heads, head_dim, 32]        (transposed, keys slot-permuted per block)
Both live in ONE allocation per tensor kind ([layers, ...]) so the cache is a single HBM
region; blocks are handed out by :class:`BlockPool` (the C++ free list in
csrc/runtime/blockpool.cpp when the runtime library is available).

Sized for the reference's LLM context (LLAMA_ARG_CTX_SIZE 4096, docker-compose.infra.yml:297) and
beyond.
"""
from __future__ import annotations

import math

import torch

from ..ops.reference import KV_BLOCK


class BlockPool:
    """LIFO free list of KV blocks (native C++ implementation with a Python fallback on CPU)."""

    def __init__(self, num_blocks: int):
        self.num_blocks = num_blocks
        self._native = None
        try:
            from ..ops._native import runtime
            lib = runtime()
            if hasattr(lib, "cfc_blockpool_create"):
                self._lib = lib
                self._native = lib.cfc_blockpool_create(num_blocks)
        except Exception:  # runtime lib not built (pure-CPU CI before build) -> python list
            self._native = None
        if self._native is None:
            self._free = list(range(num_blocks - 1, -1, -1))

    def __del__(self):
        if getattr(self, "_native", None):
            self._lib.cfc_blockpool_destroy(self._native)
            self._native = None

    def num_free(self) -> int:
        if self._native:
            return int(self._lib.cfc_blockpool_num_free(self._native))
        return len(self._free)

    def alloc(self, n: int) -> list[int]:
        if n == 0:
            return []
        if self._native:
            import numpy as np
            out = np.empty(n, dtype=np.int32)
            rc = self._lib.cfc_blockpool_alloc(self._native, n, out.ctypes.data)
            if rc != 0:
                raise MemoryError(f"KV cache exhausted: need {n} blocks, {self.num_free()} free")
            return out.tolist()
        if n > len(self._free):
            raise MemoryError(f"KV cache exhausted: need {n} blocks, {len(self._free)} free")
        out = self._free[-n:][::-1]
        del self._free[-n:]
        return out

    def free(self, blocks: list[int]) -> None:
        if not blocks:
            return
        if self._native:
            import numpy as np
            arr = np.asarray(blocks, dtype=np.int32)
            self._lib.cfc_blockpool_free(self._native, arr.ctypes.data, len(blocks))
            return
        self._free.extend(reversed(blocks))


class StateSlots:
    """Per-sequence state slots 0 .. n - 1 and one scratch slot (n): rows of a decode batch that hold no sequence, and
    a captured step's warm-up, work on the scratch."""

    def __init__(self, n: int):
        self.n, self.scratch, self._free = n, n, list(range(n - 1, -1, -1))

    def num_free(self) -> int:
        return len(self._free)

    def alloc(self, n: int) -> list[int]:
        if n > len(self._free):
            raise MemoryError(f"state slots exhausted: need {n}, {len(self._free)} free")
        return [self._free.pop() for _ in range(n)]

    def free(self, slots: list[int]) -> None:
        self._free.extend(reversed(slots))


class PagedKVCache:
    """K [layers][blocks, kv_heads, 32, D] and V^T [layers][blocks, kv_heads, D, 32] (slot-permuted,
    stored as [4 slot groups][D][8] per block and head: ops.reference.v_groups).

    ``dtype`` bf16 (default) or ``torch.float8_e4m3fn``: the FP8 cache halves the bytes the decode
    attention streams; it holds K / ``k_scale`` and V / ``v_scale`` (clamped to +-448) and the
    kernels scale back.  Opt-in: it is a precision trade-off, not the default."""

    states = None               # no state beside the blocks

    def __init__(self, layers: int, num_blocks: int, kv_heads: int, head_dim: int, device, dtype=torch.bfloat16,
                 k_scale: float = 1.0, v_scale: float = 1.0):
        if dtype not in (torch.bfloat16, torch.float8_e4m3fn):
            raise ValueError(f"KV cache dtype {dtype} not supported (bfloat16 or float8_e4m3fn)")
        self.layers, self.num_blocks, self.kv_heads, self.head_dim = layers, num_blocks, kv_heads, head_dim
        self.dtype, self.k_scale, self.v_scale = dtype, float(k_scale), float(v_scale)
        self.device = torch.device(device)
        # zero-initialised: slots of a partially filled block are read (then masked) by the kernels
        self._k = torch.zeros(layers, num_blocks, kv_heads, KV_BLOCK, head_dim, dtype=dtype, device=self.device)
        self._v = torch.zeros(layers, num_blocks, kv_heads, head_dim, KV_BLOCK, dtype=dtype, device=self.device)
        self.k = [self._k[i] for i in range(layers)]
        self.v = [self._v[i] for i in range(layers)]
        self.pool = BlockPool(num_blocks)

    @staticmethod
    def bytes_per_block(layers: int, kv_heads: int, head_dim: int, dtype_bytes: int = 2) -> int:
        return 2 * layers * kv_heads * KV_BLOCK * head_dim * dtype_bytes

    @classmethod
    def for_budget(cls, layers, kv_heads, head_dim, device, max_tokens: int, dtype=torch.bfloat16):
        nb = math.ceil(max_tokens / KV_BLOCK) + 1
        return cls(layers, nb, kv_heads, head_dim, device, dtype)

    def nbytes(self) -> int:
        return self._k.numel() * self._k.element_size() * 2


class LatentKVCache:
    """Paged cache of a latent-attention decoder, on the same blocks and :class:`BlockPool` as
    :class:`PagedKVCache`.  Per layer:
      latents [blocks, 32, rank rounded up to 32]   normed latents, pad columns zero
      tails   [blocks, slots, width] fp32           last inputs of the layer's causal convolution inside the
                                                    block, row = position % slots (None without history)
    A block holds all a sequence continuing after it needs, so prefix sharing works on whole blocks."""

    states = None
    # another sequence may map a block only after the pass that computes it (its tail is read in the
    # launch that writes tails)
    share_after_compute = True

    def __init__(self, ranks: list[int], num_blocks: int, width: int, slots: int, device, dtype=torch.bfloat16):
        self.layers, self.num_blocks, self.width, self.slots = len(ranks), num_blocks, width, slots
        self.dtype, self.device = dtype, torch.device(device)
        # zero-initialised: the slots of a partly filled block are read (then masked)
        self.latents = [torch.zeros(num_blocks, KV_BLOCK, 32 * math.ceil(r / 32), dtype=dtype, device=self.device)
                        for r in ranks]
        self.tails = [torch.zeros(num_blocks, slots, width, dtype=torch.float32, device=self.device) if slots else None
                      for _ in ranks]
        self.pool = BlockPool(num_blocks)

    def nbytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in (*self.latents, *self.tails) if t is not None)


class HybridCache:
    """Cache of a decoder whose layers are of several kinds: paged rows for those that attend, on the same blocks and
    :class:`BlockPool` as :class:`PagedKVCache`, and a state of fixed size per sequence (``states``: its slots) for
    those that recur and for what every layer remembers of the tokens before.  Per layer:
      rows   [blocks, 32, columns] or None     attention: latent and rotated key part, pad columns zero
      recur  [slots + 1, *shape] fp32 or None  recurrent state
      prev   [slots + 1, 2, width] fp32        the layer's input rows of the last two tokens, at position % 2
    A sequence's state is not in its blocks, so blocks cannot be shared between sequences.  A slot needs no clearing:
    what lies before a sequence's first token is never read."""

    share_prefix = False

    def __init__(self, columns: list[int | None], recurrent: list[tuple | None], num_blocks: int, sequences: int, width: int,
                 device, dtype=torch.bfloat16):
        self.layers, self.num_blocks, self.width = len(columns), num_blocks, width
        self.dtype, self.device = dtype, torch.device(device)
        self.states = StateSlots(sequences)
        n, f32 = sequences + 1, dict(dtype=torch.float32, device=self.device)
        # zero-initialised: the slots of a partly filled block are read (then masked)
        self.rows = [torch.zeros(num_blocks, KV_BLOCK, c, dtype=dtype, device=self.device) if c else None for c in columns]
        self.recur = [torch.zeros(n, *s, **f32) if s else None for s in recurrent]
        self.prev = [torch.zeros(n, 2, width, **f32) for _ in columns]
        self.pool = BlockPool(num_blocks)

    def nbytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in (*self.rows, *self.recur, *self.prev) if t is not None)


class PagedHeads:
    """Keys and values of one attention layer, row-major: ``k``, ``v`` [blocks, G, 32, D]; with ``pool`` the mean keys and
    values of blocks of ``pool`` tokens ``pk``, ``pv`` [blocks, G, entries, D], entry b of a sequence in block b // entries
    of its table (ops.gqa.pool_entries: allocated by the time token block b is complete)."""

    def __init__(self, num_blocks: int, heads: int, dim: int, pool: int, entries: int, device, dtype):
        def zeros(n):
            # the slots of a partly filled block are read (then masked)
            return torch.zeros(num_blocks, heads, n, dim, dtype=dtype, device=device)
        self.k, self.v, self.pool = zeros(KV_BLOCK), zeros(KV_BLOCK), pool
        self.pk, self.pv = (zeros(entries), zeros(entries)) if pool else (None, None)
        self.log2_entries = entries.bit_length() - 1 if pool else 0

    def tensors(self):
        return [t for t in (self.k, self.v, self.pk, self.pv) if t is not None]


class GroupedCache:
    """Cache of a decoder of grouped-query attention layers and recurrences, on the same blocks and :class:`BlockPool` as
    :class:`PagedKVCache`, with state slots per sequence.  Per layer (a layer that runs several times: per run):
      heads  :class:`PagedHeads`, or the very object of an earlier layer whose keys and values the layer uses, or None
      tail   [slots + 1, rows, channels] fp32 or None   last inputs of the mixer's convolution, position p at p % rows
      inputs [slots + 1, rows, width] fp32 or None      last inputs of the convolution ahead of the mixer, likewise
      recur  [slots + 1, width] fp32 or None            recurrent state
    A sequence's state is not in its blocks, so blocks cannot be shared between sequences.  A slot needs no clearing:
    what lies before a sequence's first token is never read."""

    share_prefix = False

    def __init__(self, layers: list[dict], num_blocks: int, sequences: int, device, dtype=torch.bfloat16):
        """``layers``: per layer ``heads`` (G, D, pool, entries) or the index of the layer whose it uses or None, ``tail`` and
        ``inputs`` (rows, channels) or None, ``recur`` width or None."""
        self.layers, self.num_blocks = len(layers), num_blocks
        self.dtype, self.device = dtype, torch.device(device)
        self.states = StateSlots(sequences)
        n, f32 = sequences + 1, dict(dtype=torch.float32, device=self.device)
        self.heads: list[PagedHeads | None] = []
        for c in layers:
            h = c.get("heads")
            self.heads.append(None if h is None else self.heads[h] if isinstance(h, int) else
                              PagedHeads(num_blocks, *h, self.device, dtype))
        self.tail, self.inputs = ([torch.zeros(n, *c[k], **f32) if c.get(k) else None for c in layers] for k in ("tail", "inputs"))
        self.recur = [torch.zeros(n, c["recur"], **f32) if c.get("recur") else None for c in layers]
        self.pool = BlockPool(num_blocks)

    def nbytes(self) -> int:
        rows = [t for h in {id(h): h for h in self.heads if h is not None}.values() for t in h.tensors()]
        return sum(t.numel() * t.element_size() for t in (*rows, *self.tail, *self.inputs, *self.recur) if t is not None)


def blocks_needed(n_tokens: int) -> int:
    return math.ceil(n_tokens / KV_BLOCK)
