"""Tadolix decoder: layers whose mixer is two mixers side by side -- grouped-query attention inside chunks of positions, with
capped scores and a learned bias by distance, and a minimal gated recurrence -- or a real-gated linear recurrence behind a
short convolution; a gated feed-forward or none; several copies of the stream, mixed after every sublayer; a short convolution
ahead of every mixer; a run of layers that is passed several times.

MI355X layout choices:
  * the streams, 32-bit, lie side by side per token; between two sublayers stands one kernel that sums the finished one's
    slabs, mixes the streams and norms the row the next one reads; a decoded row also goes through the mixer's input
    convolution there (ops.hyper), a prompt's rows in a pass of their own (ops.stream);
  * all projections that read one input are ONE packed matrix: a decode step takes them in one launch whose fp32 slabs the
    next kernels sum, a prompt takes each consumer's as a product of its own;
  * attention's epilogue gates its output, its factor and the recurrence's go in ahead of the activations' rounding, and both
    write side by side: the two output projections and their sum are one product (ops.gqa, ops.gru);
  * gates of the linear recurrence are block products inside its kernels, never stored (ops.rglru);
  * every pass through a layer has its own keys and values, and its own convolution inputs and recurrent states, fp32 in a
    slot per sequence;
  * tensor parallel: heads, recurrence channels (whole gate blocks), feed-forward columns and vocabulary are sharded, one
    all-reduce per sublayer.

Activations and weights are bf16, or fp32 throughout (``dtype=torch.float32``: library products and the fp32 forms of the
same kernels).
"""
from __future__ import annotations

import dataclasses
import math

import numpy as np
import torch

from ..ops import gqa as A
from ..ops import gru as R
from ..ops import hyper as X
from ..ops import kernels as K
from ..ops import rglru as L
from ..ops import stream as S
from ..ops.cols import Cols
from ..ops.reference import KV_BLOCK, interleave_gate_up
from ..runtime.kv_cache import GroupedCache
from .checkpoint import open_tensors, tensor_reader
from .decoder import argmax_keys
from .projection import JointProjection, Projection

POSITION_BASE = 10000.0                              # of the embedding's sinusoids
RATE = -8.0                                          # of the linear recurrence's log decay
GELU = dict(limit=math.inf, alpha=2.0 * math.sqrt(2.0 / math.pi), beta=0.0, cubic=0.044715)     # tanh form, as a gated sigmoid
CONV_ROWS = 32                                       # prompt rows per tile of the convolutions
DEFAULT_SEQUENCES = 256


@dataclasses.dataclass(frozen=True)
class AttnSpec:
    """Chunked attention; ``chunk`` 0: none, ``softcap`` 0: none."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float
    bias_max: float
    chunk: int
    buckets: int


@dataclasses.dataclass(frozen=True)
class ParallelSpec:
    """Attention beside a gated recurrence of ``width`` channels, each times its scale."""
    left: AttnSpec
    left_scale: float
    width: int
    right_scale: float


@dataclasses.dataclass(frozen=True)
class RgLruSpec:
    """Real-gated recurrence of ``width`` channels, gates in ``blocks``, behind ``conv`` taps."""
    width: int
    blocks: int
    conv: int


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    """``ff`` None: no feed-forward."""
    mixer: ParallelSpec | RgLruSpec
    ff: int | None


@dataclasses.dataclass(frozen=True)
class TadolixConfig:
    name: str
    vocab_size: int
    hidden: int
    specs: tuple[LayerSpec, ...]
    norm_eps: float
    taps: int
    streams: int
    embed_scale: float
    # layers loop[0] .. loop[1] - 1 run loop[2] times in a row
    loop: tuple[int, int, int] | None = None
    # nothing in the design bounds a sequence; the cache pool does
    max_positions: int = 1 << 20
    # the design names no special tokens: -1 never matches a generated one
    bos_id: int = 1
    eos_id: int = -1

    def __post_init__(self):
        if not 1 <= self.streams <= X.MAX_STREAMS:
            raise ValueError(f"{self.streams} streams (1 to {X.MAX_STREAMS})")
        if self.taps < 1:
            raise ValueError(f"input convolution of {self.taps} taps")
        if self.loop is not None and not (0 <= self.loop[0] <= self.loop[1] <= len(self.specs) and self.loop[2] >= 1):
            raise ValueError(f"loop {self.loop} over {len(self.specs)} layers")
        for i, s in enumerate(self.specs):
            m = s.mixer
            if isinstance(m, RgLruSpec) and (m.width % m.blocks or m.conv < 1):
                raise ValueError(f"layer {i}: {m.width} channels in {m.blocks} blocks, {m.conv} taps")
            if isinstance(m, ParallelSpec) and m.left.heads % m.left.kv_heads:
                raise ValueError(f"layer {i}: {m.left.heads} heads on {m.left.kv_heads}")

    @property
    def layers(self) -> int:
        return len(self.specs)

    @property
    def runs(self) -> tuple[int, ...]:
        """Layers in the order they run."""
        n, (a, b, times) = len(self.specs), self.loop or (0, 0, 1)
        return (*range(a), *(tuple(range(a, b)) * times), *range(b, n))

    def num_params(self) -> int:
        return sum(math.prod(s) for s in TadolixWeights.tensor_shapes(self).values())

    def flops_per_token(self, ctx: int = 0) -> float:
        """Product flops per token (+ attention over what ``ctx`` tokens leave to see)."""
        W = self.hidden
        f = 2.0 * W * self.vocab_size
        for i in self.runs:
            m, ff = self.specs[i].mixer, self.specs[i].ff
            if isinstance(m, ParallelSpec):
                a = m.left
                f += 2 * W * (a.heads * (a.dim + 2 * a.vdim) + a.kv_heads * (a.dim + a.vdim) + 4 * m.width)
                f += 2 * a.heads * (a.dim + a.vdim) * (min(ctx, a.chunk) if a.chunk else ctx)
            else:
                f += 6 * W * m.width + 4 * m.width * (m.width // m.blocks)
            f += 6 * W * (ff or 0)
        return f


def config_from_json(c: dict, name: str = "tadolix", ckpt_dir=None) -> TadolixConfig:
    """TadolixConfig from a parsed config.json and (``ckpt_dir``) the shapes of the tensors beside it: the rows of the distance
    biases stand nowhere else."""
    tensors, specs = None, []
    for i, layer in enumerate(c["layers"]):
        m, f, kind = layer["mixer"], layer.get("mlp"), layer["type"]
        if kind == "parallel":
            a, rows = m["left"], m["left"].get("buckets")
            if rows is None and ckpt_dir is not None:
                tensors = tensors or open_tensors(ckpt_dir)
                rows = tensors[f"l{i}.mix.left.rel"].get_slice(f"l{i}.mix.left.rel").get_shape()[0]
            if rows is None:
                raise ValueError(f"layer {i}: the rows of the distance bias are not in config.json: give the tensors' folder")
            mixer = ParallelSpec(AttnSpec(int(a["heads"]), int(a["kv_heads"]), int(a["dim"]), int(a["vdim"]), float(a["scale"]),
                                          float(a.get("softcap") or 0.0), float(a["bias_max"]), int((a.get("mask") or {}).get("size") or 0),
                                          int(rows)),
                                 float(m["left_scale"]), int(m["right"]["width"]), float(m["right_scale"]))
        elif kind == "rglru":
            mixer = RgLruSpec(int(m["width"]), int(m["blocks"]), int(m["conv"]))
        else:
            raise NotImplementedError(f"layer {i}: mixer {kind!r} (Tadolix has parallel and rglru)")
        if f is not None and f["kind"] != "dense":
            raise NotImplementedError(f"layer {i}: feed-forward {f['kind']!r} (Tadolix has dense)")
        specs.append(LayerSpec(mixer, int(f["ff"]) if f is not None else None))
    loop = c.get("loop")
    return TadolixConfig(name, int(c["vocab"]), int(c["width"]), tuple(specs), float(c["norm"]["eps"]), int(c["canon"]["taps"]),
                         int(c["streams"]), float(c["embedding"]["scale"]),
                         (int(loop["start"]), int(loop["stop"]), int(loop["times"])) if loop else None)


def pattern_config(name: str, vocab: int, hidden: int, layers: int, par: ParallelSpec, lru: RgLruSpec, ff: int, taps: int = 4,
                   streams: int = 4, loop=None, eps: float = 1e-6, max_positions: int = 1 << 20) -> TadolixConfig:
    """Both kinds of layers in turn, every second recurrent one without feed-forward."""
    specs = tuple(LayerSpec(lru if i % 2 else par, None if i % 4 == 1 else ff) for i in range(layers))
    return TadolixConfig(name, vocab, hidden, specs, eps, taps, streams, hidden ** 0.5, loop, max_positions)


PRESETS: dict[str, TadolixConfig] = {
    # Mistral-7B's width, depth, heads and feed-forward
    "tadolix-7b": pattern_config(
        "tadolix-7b", 32000, 4096, 32, ParallelSpec(AttnSpec(32, 8, 128, 128, 128 ** -0.5, 50.0, 256, 2048, 32), 0.7, 4096, 0.7),
        RgLruSpec(4096, 16, 4), 14336, max_positions=32768),
    "tadolix-small": pattern_config(
        "tadolix-small", 32000, 1024, 4, ParallelSpec(AttnSpec(16, 4, 64, 64, 0.125, 30.0, 128, 512, 32), 0.7, 1024, 0.7),
        RgLruSpec(1024, 8, 4), 2816, max_positions=8192),
    "tiny-tadolix": pattern_config(
        "tiny-tadolix", 512, 128, 4, ParallelSpec(AttnSpec(4, 2, 32, 48, 0.3, 20.0, 60, 40, 12), 0.9, 96, 0.6),
        RgLruSpec(120, 3, 3), 192, taps=3, streams=3, loop=(1, 3, 2), max_positions=4096),
}


def get_config(name_or_cfg) -> TadolixConfig:
    return name_or_cfg if isinstance(name_or_cfg, TadolixConfig) else PRESETS[name_or_cfg]


class TadolixWeights:
    """Per-rank (TP-sharded) weights on one device: matrices in ``dtype``, vectors in fp32."""

    def __init__(self, cfg: TadolixConfig, device, tp_rank: int = 0, tp_size: int = 1, dtype=torch.bfloat16):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"Tadolix weights in bfloat16 or float32, not {dtype}")
        sharded = [cfg.vocab_size]
        for s in cfg.specs:
            m = s.mixer
            sharded += [m.left.heads, m.left.kv_heads, m.width] if isinstance(m, ParallelSpec) else [m.blocks]
            sharded.append(s.ff or 0)
        if any(n % tp_size for n in sharded):
            raise ValueError(f"{cfg.name}: heads / recurrence width and blocks / ff / vocab must divide tp_size={tp_size}")
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.tp_rank, self.tp_size = tp_rank, tp_size
        self.vocab_shard = cfg.vocab_size // tp_size
        self.layers: list[dict] = []
        self.embed = self.head = self.final_norm = self.turns = None

    @staticmethod
    def tensor_shapes(cfg: TadolixConfig) -> dict[str, tuple]:
        """Every tensor of a checkpoint and its shape."""
        W, n = cfg.hidden, cfg.streams
        out = {"embed": (cfg.vocab_size, W), "head": (cfg.vocab_size, W), "final.norm": (W,)}
        for i, s in enumerate(cfg.specs):
            m, p = s.mixer, f"l{i}."
            x = p + "mix."
            for q in (1, 2) if s.ff is not None else (1,):
                out |= {f"{p}norm{q}": (W,), f"{p}hc{q}.in": (n,), f"{p}hc{q}.out": (n,), f"{p}hc{q}.mix": (n, n)}
            out[p + "canon1"] = (W, cfg.taps)
            if isinstance(m, ParallelSpec):
                a, C = m.left, m.width
                y = x + "right."
                out |= {x + "left." + k: (h, W) for k, h in (("q", a.heads * a.dim), ("k", a.kv_heads * a.dim), ("v", a.kv_heads * a.vdim),
                                                             ("g", a.heads * a.vdim))}
                out |= {x + "left.rel": (a.buckets, a.heads), x + "left.o": (W, a.heads * a.vdim)}
                out |= {y + k: (C, W) for k in "zxg"} | {y + "z.b": (C,), y + "x.b": (C,), y + "o": (W, C)}
            else:
                C, b = m.width, m.width // m.blocks
                out |= {x + "y": (C, W), x + "y.b": (C,), x + "x": (C, W), x + "x.b": (C,), x + "conv": (C, m.conv), x + "conv.b": (C,),
                        x + "lam": (C,), x + "o": (W, C)}
                out |= {x + k: (m.blocks, b, b) for k in ("ra", "ri")} | {x + k + ".b": (m.blocks, b) for k in ("ra", "ri")}
            if s.ff is not None:
                out |= {p + "mlp.gate": (s.ff, W), p + "mlp.up": (s.ff, W), p + "mlp.down": (W, s.ff)}
        return out

    @classmethod
    def from_safetensors(cls, cfg, ckpt_dir, device, tp_rank: int = 0, tp_size: int = 1, dtype=torch.bfloat16):
        return cls._build(cfg, tensor_reader(ckpt_dir, cls.tensor_shapes(cfg)), device, tp_rank, tp_size, dtype)

    @classmethod
    def random(cls, cfg, device, seed: int = 0, tp_rank: int = 0, tp_size: int = 1, std: float = 0.02,
               dtype=torch.bfloat16):
        """Random weights of the full model, drawn tensor by tensor on the device (every TP rank draws the
        same full tensors and keeps its shard)."""
        dev = torch.device(device)
        gen = torch.Generator(device=dev)
        gen.manual_seed(seed * 1000003 + 99)
        shapes = cls.tensor_shapes(cfg)

        def get(name):
            t = torch.empty(shapes[name], dtype=torch.float32, device=dev)
            kind = name.rsplit(".", 1)[-1]
            if kind.startswith("norm"):
                return t.normal_(0.0, 0.1, generator=gen)
            if kind == "in":
                return t.fill_(1.0 / cfg.streams)
            if kind == "out":
                return t.fill_(1.0)
            if kind == "mix":
                return t.fill_(0.1 / cfg.streams) + 0.9 * torch.eye(cfg.streams, device=dev)
            if kind == "lam":
                return t.uniform_(-5.0, -1.0, generator=gen)
            if kind in ("b", "conv", "rel") or kind.startswith("canon"):
                return t.normal_(0.0, 0.2 if kind.startswith("canon") else 0.5, generator=gen)
            scale = 1.0 / math.sqrt(shapes[name][2]) if kind in ("ra", "ri") else 1.0 / math.sqrt(cfg.hidden) if name == "embed" else std
            return t.normal_(0.0, scale, generator=gen).to(torch.bfloat16)
        return cls._build(cfg, get, dev, tp_rank, tp_size, dtype)

    @classmethod
    def _build(cls, cfg, get, device, tp_rank, tp_size, dtype):
        w = cls(cfg, device, tp_rank, tp_size, dtype)

        def mat(t):
            return t.to(device=w.device, dtype=w.dtype)

        def vec(t):
            return t.to(device=w.device, dtype=torch.float32).contiguous()

        def rows(t):
            return t.view(tp_size, t.shape[0] // tp_size, *t.shape[1:])[tp_rank]

        def cols(t):
            return t.view(t.shape[0], tp_size, t.shape[1] // tp_size)[:, tp_rank].contiguous()

        for i, s in enumerate(cfg.specs):
            m, p, x = s.mixer, f"l{i}.", f"l{i}.mix."
            lw = {"norm1": 1.0 + vec(get(p + "norm1")), "canon": vec(get(p + "canon1")).t().contiguous()}
            for q in (1, 2) if s.ff is not None else (1,):
                lw[f"hc{q}"] = X.Connection(*(vec(get(f"{p}hc{q}.{k}")) for k in ("in", "mix", "out")))
            if isinstance(m, ParallelSpec):
                a, y = m.left, x + "right."
                ones = torch.ones(a.dim, dtype=torch.float32, device=w.device)
                bias = A.distance_bias(cols(vec(get(x + "left.rel"))), a.bias_max, a.chunk)
                lw["heads"] = A.Heads(a.heads // tp_size, a.kv_heads // tp_size, a.dim, a.vdim, a.scale, A.Mask(a.chunk, chunked=a.chunk > 0),
                                      cfg.norm_eps, ones, ones, True, None, softcap=a.softcap, bias=bias, unit=True)
                lw["gru"] = R.Gru(vec(rows(get(y + "z.b"))), vec(rows(get(y + "x.b"))))
                lw["in"] = JointProjection([(mat(torch.cat([rows(get(x + "left." + k)) for k in "qkv"])), 0),
                                            (mat(torch.cat([rows(get(y + k)) for k in "zxg"])), 0), (mat(rows(get(x + "left.g"))), 0)])
                lw["o"] = Projection(torch.cat([mat(cols(get(x + "left.o"))), mat(cols(get(y + "o")))], 1))
            else:
                lw["lru"] = L.RgLru(vec(rows(get(x + "x.b"))), vec(rows(get(x + "conv"))).t().contiguous(), vec(rows(get(x + "conv.b"))),
                                    mat(rows(get(x + "ra"))), vec(rows(get(x + "ra.b"))).view(-1), mat(rows(get(x + "ri"))),
                                    vec(rows(get(x + "ri.b"))).view(-1),
                                    (RATE * torch.nn.functional.softplus(rows(get(x + "lam")).double())).float().to(w.device),
                                    vec(rows(get(x + "y.b"))))
                lw["in"] = JointProjection([(mat(torch.cat([rows(get(x + k)) for k in "yx"])), 0)])
                lw["o"] = Projection(mat(cols(get(x + "o"))))
            if s.ff is not None:
                lw["norm2"] = 1.0 + vec(get(p + "norm2"))
                gu = torch.cat([mat(rows(get(p + "mlp.gate"))), mat(rows(get(p + "mlp.up")))])
                lw["interleaved"] = (s.ff // tp_size) % 8 == 0
                fused = lw["interleaved"] and Projection.packs(gu, gu.shape[0], cfg.hidden)
                lw["gate_up"] = Projection(interleave_gate_up(gu) if lw["interleaved"] else gu, swiglu=fused)
                lw["down"] = Projection(mat(cols(get(p + "mlp.down"))))
            w.layers.append(lw)
        w.embed = mat(get("embed")).contiguous()
        w.head = Projection(mat(rows(get("head"))))
        w.final_norm = 1.0 + vec(get("final.norm"))
        w.turns = S.sinusoid_turns(cfg.hidden, POSITION_BASE, w.device)
        if w.device.type == "cuda":
            torch.cuda.empty_cache()
        return w

    def nbytes(self) -> int:
        n = self.embed.numel() * self.embed.element_size() + self.head.nbytes()
        return n + sum(lw[k].nbytes() for lw in self.layers for k in ("in", "o", "lru", "gate_up", "down") if k in lw)


@dataclasses.dataclass
class _Pass:
    """What a pass over packed rows goes by: a decode step (one token per sequence, P key slices) or, with ``plan``,
    portions of prompts."""
    positions: torch.Tensor
    slots: torch.Tensor
    states: torch.Tensor
    ctx_lens: torch.Tensor
    block_tables: torch.Tensor
    kv: GroupedCache
    plan: dict | None = None
    cu_q: torch.Tensor | None = None
    P: int = 1
    workspace: torch.Tensor | None = None


class TadolixModel:
    """Stateless forward functions over :class:`TadolixWeights` + a :class:`GroupedCache`."""

    @staticmethod
    def kernel_sources(cfg, dtype) -> tuple:
        """csrc/kernels sources a run of this configuration launches kernels from."""
        src = {"elementwise", "stream", "hyper"}
        for s in cfg.specs:
            src |= {"qkv", "gqa", "gru"} if isinstance(s.mixer, ParallelSpec) else {"rglru"}
        if dtype == torch.bfloat16:
            src |= {"gemm", "dgemm", "pgemm"}
        return tuple(sorted(src))

    def __init__(self, weights: TadolixWeights, tp_group=None, custom_ar=None):
        self.w = weights
        self.cfg = weights.cfg
        self.tp_group = tp_group
        self.custom_ar = custom_ar

    # ---------------------------------------------------------------- engine interface
    def new_cache(self, num_blocks: int, dtype=None, device=None, sequences: int | None = None) -> GroupedCache:
        if dtype not in (None, self.w.dtype):
            raise ValueError(f"cache in the model's dtype ({self.w.dtype}), not {dtype}")
        layers, taps = [], self.cfg.taps
        for lw in (self.w.layers[i] for i in self.cfg.runs):
            c = {"inputs": (taps - 1, self.cfg.hidden) if taps > 1 else None}
            if "heads" in lw:
                c |= {"heads": (lw["heads"].G, lw["heads"].D, 0, 0), "recur": lw["gru"].width}
            else:
                c |= {"tail": (lw["lru"].ring, lw["lru"].width), "recur": lw["lru"].width}
            layers.append(c)
        return GroupedCache(layers, num_blocks, sequences or min(num_blocks, DEFAULT_SEQUENCES), device or self.w.device, self.w.dtype)

    def _heads(self):
        return [lw["heads"] for lw in self.w.layers if "heads" in lw]

    def decode_partitions(self, B: int, max_blocks: int) -> int:
        """Key slices per sequence of a B-row decode step over block tables ``max_blocks`` wide."""
        ctx = max_blocks * KV_BLOCK
        return max([1] + [A.decode_slices(B, a.H, a.G, a.D, a.mask.visible(ctx), self.w.dtype) for a in self._heads()])

    def decode_workspace(self, B: int, P: int) -> int:
        return max([1] + [B * a.H * P * (a.D + 2) for a in self._heads()]) if P > 1 else 1

    def _tiles(self, a: A.Heads) -> str:
        return f"tiles_{a.H}_{a.G}_{A.prompt_rows(self.w.dtype, a.D)}"

    def plan_prefill(self, cu, ctx, slots, states) -> dict:
        """Host-side launch plan of a packed pass over portions cu / ctx in state slots ``states``: int32 arrays for
        the device."""
        n = np.diff(np.asarray(cu))
        portions = [(int(a), int(k), int(c - k), s) for s, (a, k, c) in enumerate(zip(cu, n, ctx))]
        rows = max([CONV_ROWS, self.cfg.taps - 1] + [lw["lru"].taps - 1 for lw in self.w.layers if "lru" in lw])
        plan = {"states": np.asarray(states, np.int32), "row_states": np.repeat(np.asarray(states, np.int32), n),
                "lead": np.concatenate([np.arange(k, dtype=np.int32) for k in n]), "conv_tiles": S.conv_tiles(portions, rows)}
        for lw in self.w.layers:
            if "heads" in lw:
                a = lw["heads"]
                if self._tiles(a) not in plan:
                    plan[self._tiles(a)] = A.prompt_tiles(cu, ctx, a.H, a.G, A.prompt_rows(self.w.dtype, a.D))
                if "chunks" not in plan:
                    plan["chunks"], plan["chunk_cu"] = R.chunk_plan(cu)
            elif "segments" not in plan and not L.whole_portions(cu, lw["lru"].width):
                plan["segments"], plan["segment_cu"] = R.chunk_plan(cu, L.SEGMENT)
        return plan

    # ---------------------------------------------------------------- forward
    def forward_prefill(self, ids, positions, slots, cu_q, ctx_lens, block_tables, kv, last_idx=None, plan=None):
        """Packed portions of prompts (down to one token each), their launch plan from :meth:`plan_prefill`.  Returns
        the final-normed hidden states of rows ``last_idx`` (or all rows)."""
        return self._layers(ids, _Pass(positions, slots, plan["states"], ctx_lens, block_tables, kv, plan, cu_q),
                            None if last_idx is None else last_idx.to(torch.int32))

    def forward_decode(self, ids, positions, slots, ctx_lens, block_tables, kv, attn_workspace=None, part_blocks=-1,
                       shared_blocks=None, states=None):
        """One token per sequence, ``states`` their state slots.  Returns the final-normed hidden states [B, W].
        ``part_blocks``: -P, P key slices per sequence (the engine's form); ``shared_blocks`` is not used."""
        return self._layers(ids, _Pass(positions, slots, states, ctx_lens, block_tables, kv, P=max(1, -part_blocks),
                                       workspace=attn_workspace))

    def _layers(self, ids, io: _Pass, rows=None) -> torch.Tensor:
        T, W, dt, eps, dev = ids.numel(), self.cfg.hidden, self.w.dtype, self.cfg.norm_eps, ids.device
        e = S.embed_f32(self.w.embed, ids, torch.empty(T, W, dtype=torch.float32, device=dev), self.cfg.embed_scale, io.positions,
                        self.w.turns)
        xs = X.Streams(e, self.cfg.streams)
        h = torch.empty(T, W, dtype=dt, device=dev)
        u, rstd = (torch.empty(T, W, dtype=torch.float32, device=dev), torch.empty(T, dtype=torch.float32, device=dev)) \
            if io.plan is not None else (None, None)
        for run, i in enumerate(self.cfg.runs):
            lw = self.w.layers[i]
            c, tail = lw["hc1"], S.Tail(io.kv.inputs[run], io.states)
            if io.plan is None:
                X.conv_decode(xs, c.inp, lw["norm1"], eps, lw["canon"], io.positions, tail, h)
            else:
                X.stats(xs, c.inp, eps, u, rstd)
                S.input_conv(u, rstd, lw["norm1"], [lw["canon"]], io.plan["conv_tiles"], tail, [h])
            xs.done = self._mixer(i, run, h, io), c
            if "hc2" in lw:
                c = lw["hc2"]
                X.norm(xs, c.inp, lw["norm2"], eps, h)
                xs.done = self._feed(i, h), c
        return X.last_norm(xs, self.w.final_norm, eps, dt, rows)

    def _mixer(self, i, run, h, io: _Pass) -> torch.Tensor:
        """fp32 slabs [split, T, W] of layer i's mixer."""
        lw, m = self.w.layers[i], self.cfg.specs[i].mixer
        hs = h[None]
        c = lw["in"].joint(hs) if io.plan is None else [lw["in"].act(j, hs) for j in range(len(lw["in"].sizes))]
        if "lru" in lw:
            return self._sum(lw["o"].slabs(self._lru(lw["lru"], run, c[0], io)))
        a, n = lw["heads"], lw["gru"].width
        both = torch.empty(h.shape[0], a.H * a.vdim + n, dtype=self.w.dtype, device=h.device)
        self._recur(lw["gru"], run, c[1], io, m.right_scale, both[:, a.H * a.vdim:])
        self._attend(a, run, c[0], c[2], io, m.left_scale, both[:, :a.H * a.vdim])
        return self._sum(lw["o"].slabs(both))

    def _attend(self, a: A.Heads, run, cols: Cols, gate: Cols, io: _Pass, factor, out) -> None:
        rows = io.kv.heads[run]
        if io.plan is None:
            q = A.qkv_rows(a, cols, rows, io.positions, io.slots, io.states, io.block_tables)
            A.attention(a, q, rows, io.block_tables, io.ctx_lens, P=io.P, workspace=io.workspace, gate=gate, factor=factor, out=out)
            return
        p = io.plan
        q = A.qkv_rows(a, cols, rows, io.positions, io.slots, p["row_states"], io.block_tables, None, p["lead"])
        A.attention(a, q, rows, io.block_tables, io.ctx_lens, io.cu_q, p[self._tiles(a)], gate=gate, factor=factor, out=out)

    def _recur(self, g: R.Gru, run, cols: Cols, io: _Pass, factor, out) -> None:
        state = io.kv.recur[run]
        zxg = [Cols(cols.t, cols.c0 + k * g.width, g.width) for k in range(3)]
        if io.plan is None:
            R.step(g, *zxg, io.states, io.ctx_lens, state, out, factor)
        else:
            R.prefill(g, *zxg, io.states, io.cu_q, io.ctx_lens, io.plan["chunks"], io.plan["chunk_cu"], state, out, factor)

    def _lru(self, r: L.RgLru, run, cols: Cols, io: _Pass) -> torch.Tensor:
        y, x = (Cols(cols.t, cols.c0 + k * r.width, r.width) for k in range(2))
        out = torch.empty(cols.rows, r.width, dtype=self.w.dtype, device=cols.t.device)
        tail, state, p = io.kv.tail[run], io.kv.recur[run], io.plan
        if p is None:
            return L.step(r, x, y, io.states, io.positions, io.ctx_lens, tail, state, out)
        # a pass that has segments for one layer's width runs all layers on them
        return L.prefill(r, x, y, io.states, io.cu_q, io.ctx_lens, p["conv_tiles"], p.get("segments"), p.get("segment_cu"), tail, state, out)

    def _feed(self, i, h) -> torch.Tensor:
        """fp32 slabs of layer i's feed-forward."""
        lw = self.w.layers[i]
        a = torch.empty(h.shape[0], lw["down"].K, dtype=h.dtype, device=h.device)
        if lw["interleaved"]:
            lw["gate_up"].glu(h, a, **GELU)
        else:
            S.clamped_glu(lw["gate_up"].slabs(h), a, **GELU)
        return self._sum(lw["down"].slabs(a))

    def _sum(self, slabs) -> torch.Tensor:
        """A sharded product's slabs as one all-reduced slab (TP), else as they are."""
        if self.w.tp_size == 1:
            return slabs
        part = slabs[:1].clone()
        for p in slabs[1:]:                # elementwise adds: nothing a captured graph could not hold
            part.add_(p)
        torch.distributed.all_reduce(part, group=self.tp_group)
        return part

    # ---------------------------------------------------------------- output
    def logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """[B, V] fp32 logits (all-gathered over the vocabulary shards)."""
        local = self.w.head.f32(hidden)
        if self.w.tp_size == 1:
            return local
        parts = [torch.empty_like(local) for _ in range(self.w.tp_size)]
        torch.distributed.all_gather(parts, local, group=self.tp_group)
        return torch.cat(parts, -1)

    def greedy_ids(self, hidden: torch.Tensor, out: torch.Tensor) -> torch.Tensor:
        """Greedy next tokens into ``out``; under TP the shards' argmax keys are reduced instead of
        gathering the logits."""
        local = self.w.head.f32(hidden)
        if self.w.tp_size == 1:
            return K.sample(local, out, 0.0)
        keys = argmax_keys(local, self.w.tp_rank * self.w.vocab_shard)
        torch.distributed.all_reduce(keys, op=torch.distributed.ReduceOp.MAX, group=self.tp_group)
        out.copy_((0xFFFFFFFF - (keys & 0xFFFFFFFF)).to(torch.int32))
        return out

    def graph_collectives_ok(self, B: int) -> bool:
        return self.w.tp_size == 1
