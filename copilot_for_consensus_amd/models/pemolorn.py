"""Pemolorn decoder: layers whose mixer is grouped-query attention over a window and the kept first tokens, or two mixers
side by side -- attention over a window and pooled blocks behind it, and a minimal gated recurrence -- with a dense
(squared relu) or a routed feed-forward, some of whose choices are the identity, or none; a scalar-gained RMS norm on
either side of every sublayer.

MI355X layout choices:
  * keys and values are cached row-major per key head, the means of pooled blocks beside them in the same paged blocks;
    a far block costs one row, so decode streams window + context / pool rows, and a layer that uses another's keys holds
    none.  Convolution inputs and recurrent state are fp32 in a slot per sequence;
  * all projections that read one input are ONE packed matrix: a decode step takes them in one launch whose fp32 slabs
    the next kernels sum, a prompt takes attention's and the recurrence's as a product each;
  * convolution, norm, rotation, cache write and (decode) pooling are one kernel (ops.gqa); between two sublayers stands
    one kernel that sums slabs or expert rows, norms the branch, adds it and norms the next input (ops.branch);
  * prompt portions of the recurrence run chunk-parallel (ops.gru); experts are routed and sorted on the device (ops.moe);
  * tensor parallel: attention heads, recurrence channels, feed-forward columns (each expert's too) and vocabulary are
    sharded, routers replicated; the attention beside a recurrence is replicated, as its norms run over all heads.  One
    all-reduce per sublayer.

Activations and weights are bf16, or fp32 throughout (``dtype=torch.float32``: library products and the fp32 forms of the
same kernels).
"""
from __future__ import annotations

import dataclasses
import math

import numpy as np
import torch

from ..ops import branch as N
from ..ops import gqa as A
from ..ops import gru as R
from ..ops import kernels as K
from ..ops import moe as M
from ..ops import stream as S
from ..ops.cols import Cols
from ..ops.reference import KV_BLOCK
from ..runtime.kv_cache import GroupedCache
from .checkpoint import tensor_reader
from .decoder import argmax_keys
from .projection import JointProjection, Projection

GLU_ALPHA = 1.702     # slope of the experts' gate sigmoid
GLU_SHIFT = 1.0       # added to their clamped up projection
DEFAULT_SEQUENCES = 256


@dataclasses.dataclass(frozen=True)
class AttnSpec:
    """Attention of one layer.  ``conv`` taps over time ahead of the norms (0: none), ``rot`` rotated dimensions;
    ``kv_from``: the layer whose keys and values it uses."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    mask: A.Mask
    conv: int = 0
    rot: int = 0
    base: float = 1.0
    kv_from: int | None = None


@dataclasses.dataclass(frozen=True)
class ParallelSpec:
    """Attention beside a recurrence of ``width`` channels."""
    left: AttnSpec
    width: int


@dataclasses.dataclass(frozen=True)
class DenseSpec:
    ff: int


@dataclasses.dataclass(frozen=True)
class MoeSpec:
    """Routed experts of ``ff``, beside ``identity`` choices without matrices."""
    ff: int
    limit: float
    experts: int
    identity: int
    top: int


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: AttnSpec | ParallelSpec
    mlp: DenseSpec | MoeSpec | None

    @property
    def attn(self) -> AttnSpec:
        return self.mixer.left if isinstance(self.mixer, ParallelSpec) else self.mixer


@dataclasses.dataclass(frozen=True)
class PemolornConfig:
    name: str
    vocab_size: int
    hidden: int
    specs: tuple[LayerSpec, ...]
    norm_eps: float
    # nothing in the design bounds a sequence; the cache pool does
    max_positions: int = 1 << 20
    # the design names no special tokens: -1 never matches a generated one
    bos_id: int = 1
    eos_id: int = -1

    def __post_init__(self):
        for i, s in enumerate(self.specs):
            a = s.attn
            if a.kv_from is None:
                continue
            if not 0 <= a.kv_from < i:
                raise ValueError(f"layer {i}: keys of layer {a.kv_from}, which does not come before it")
            o = self.specs[a.kv_from]
            if isinstance(o.mixer, ParallelSpec) or o.attn.kv_from is not None or \
                    (o.attn.kv_heads, o.attn.dim, o.attn.vdim) != (a.kv_heads, a.dim, a.vdim):
                raise ValueError(f"layer {i}: layer {a.kv_from} has no keys and values of its shape")

    @property
    def layers(self) -> int:
        return len(self.specs)

    def num_params(self) -> int:
        return sum(math.prod(s) for s in PemolornWeights.tensor_shapes(self).values())

    def flops_per_token(self, ctx: int = 0) -> float:
        """Product flops per token (chosen experts only; + attention over what ``ctx`` tokens leave to see)."""
        W = self.hidden
        f = 2.0 * W * self.vocab_size
        for s in self.specs:
            a, p = s.attn, s.mlp
            kv = 0 if a.kv_from is not None else a.kv_heads * (a.dim + a.vdim)
            f += 2 * W * (a.heads * (a.dim + a.vdim) + kv) + 2 * a.heads * (a.dim + a.vdim) * a.mask.visible(ctx)
            if isinstance(s.mixer, ParallelSpec):
                f += 8 * W * s.mixer.width
            if isinstance(p, DenseSpec):
                f += 4 * W * p.ff
            elif p is not None:
                f += 6 * W * p.ff * p.top * p.experts / (p.experts + p.identity) + 2 * W * (p.experts + p.identity)
        return f


def _attn_from_json(m: dict) -> AttnSpec:
    mask, rot = m.get("mask") or {}, m.get("rot") or {}
    kv = m.get("kv_from")
    return AttnSpec(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), float(m["scale"]),
                    A.Mask(int(mask.get("size") or 0), int(mask.get("keep_first") or 0), int(mask.get("pool") or 0)),
                    int(m.get("conv") or 0), int(rot.get("dims") or 0), float(rot.get("base", 1.0)), None if kv is None else int(kv))


def config_from_json(c: dict, name: str = "pemolorn") -> PemolornConfig:
    """PemolornConfig from a parsed config.json."""
    specs = []
    for i, layer in enumerate(c["layers"]):
        m, f, kind = layer["mixer"], layer.get("mlp"), layer["type"]
        if kind == "attention":
            if m.get("conv") or m.get("rot"):
                raise NotImplementedError(f"layer {i}: convolution or rotation in an attention layer")
            mixer = _attn_from_json(m)
        elif kind == "parallel":
            if m["left"].get("kv_from") is not None:
                raise NotImplementedError(f"layer {i}: shared keys beside a recurrence")
            mixer = ParallelSpec(_attn_from_json(m["left"]), int(m["right"]["width"]))
        else:
            raise NotImplementedError(f"layer {i}: mixer {kind!r} (Pemolorn has attention and parallel)")
        if f is None:
            mlp = None
        elif f["kind"] == "dense":
            mlp = DenseSpec(int(f["ff"]))
        elif f["kind"] == "moe":
            r = f["router"]
            mlp = MoeSpec(int(f["expert"]["ff"]), float(f["expert"]["limit"]), int(r["experts"]), int(r.get("identity") or 0), int(r["top"]))
        else:
            raise NotImplementedError(f"layer {i}: feed-forward {f['kind']!r} (Pemolorn has dense and moe)")
        specs.append(LayerSpec(mixer, mlp))
    return PemolornConfig(name, int(c["vocab"]), int(c["width"]), tuple(specs), float(c["norm"]["eps"]))


def pattern_config(name: str, vocab: int, hidden: int, layers: int, attn: AttnSpec, par: ParallelSpec, dense: DenseSpec, moe: MoeSpec,
                   eps: float = 1e-6, max_positions: int = 1 << 20) -> PemolornConfig:
    """Runs of four layers: attention, attention beside a recurrence, attention on the first one's keys, and another
    parallel one; dense and routed feed-forwards in turn."""
    specs = []
    for i in range(layers):
        own = attn if i % 4 != 2 else dataclasses.replace(attn, kv_from=i - 2)
        specs.append(LayerSpec(par if i % 2 else own, moe if i % 2 else dense))
    return PemolornConfig(name, vocab, hidden, tuple(specs), eps, max_positions)


PRESETS: dict[str, PemolornConfig] = {
    # Mistral-7B's width, depth, heads and feed-forward
    "pemolorn-7b": pattern_config(
        "pemolorn-7b", 32000, 4096, 32, AttnSpec(32, 8, 128, 128, 128 ** -0.5, A.Mask(4096, keep=4)),
        ParallelSpec(AttnSpec(32, 8, 128, 128, 128 ** -0.5, A.Mask(1024, pool=16), conv=4, rot=64, base=1e6), 4096),
        DenseSpec(14336), MoeSpec(1024, 7.0, 32, 4, 4), max_positions=32768),
    "pemolorn-small": pattern_config(
        "pemolorn-small", 32000, 1024, 4, AttnSpec(16, 4, 64, 64, 0.125, A.Mask(1024, keep=4)),
        ParallelSpec(AttnSpec(8, 4, 96, 96, 96 ** -0.5, A.Mask(256, pool=8), conv=4, rot=32, base=1e5), 1024),
        DenseSpec(4096), MoeSpec(512, 7.0, 16, 2, 2), max_positions=8192),
    "tiny-pemolorn": pattern_config(
        "tiny-pemolorn", 512, 128, 4, AttnSpec(4, 2, 32, 48, 0.2, A.Mask(50, keep=3)),
        ParallelSpec(AttnSpec(2, 1, 40, 32, 0.15, A.Mask(24, pool=6), conv=3, rot=16, base=5000.0), 96),
        DenseSpec(192), MoeSpec(64, 3.0, 6, 2, 3), max_positions=4096),
}


def get_config(name_or_cfg) -> PemolornConfig:
    return name_or_cfg if isinstance(name_or_cfg, PemolornConfig) else PRESETS[name_or_cfg]


class PemolornWeights:
    """Per-rank (TP-sharded) weights on one device: matrices in ``dtype``, vectors in fp32."""

    def __init__(self, cfg: PemolornConfig, device, tp_rank: int = 0, tp_size: int = 1, dtype=torch.bfloat16):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"Pemolorn weights in bfloat16 or float32, not {dtype}")
        sharded = [cfg.vocab_size]
        for s in cfg.specs:
            sharded += [s.mixer.width] if isinstance(s.mixer, ParallelSpec) else [s.mixer.heads, s.mixer.kv_heads]
            if s.mlp is not None:
                sharded.append(s.mlp.ff)
        if any(n % tp_size for n in sharded):
            raise ValueError(f"{cfg.name}: heads / recurrence width / ff / vocab must divide tp_size={tp_size}")
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.tp_rank, self.tp_size = tp_rank, tp_size
        self.vocab_shard = cfg.vocab_size // tp_size
        self.layers: list[dict] = []
        self.embed = self.head = self.final_norm = None

    @staticmethod
    def tensor_shapes(cfg: PemolornConfig) -> dict[str, tuple]:
        """Every tensor of a checkpoint and its shape."""
        W = cfg.hidden
        out = {"embed": (cfg.vocab_size, W), "head": (cfg.vocab_size, W), "final.norm": ()}
        for i, s in enumerate(cfg.specs):
            a, f, p = s.attn, s.mlp, f"l{i}."
            par = isinstance(s.mixer, ParallelSpec)
            x = p + ("mix.left." if par else "mix.")
            sizes = {"q": a.heads * a.dim} | ({} if a.kv_from is not None else {"k": a.kv_heads * a.dim, "v": a.kv_heads * a.vdim})
            out |= {p + n: () for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f is not None else ())}
            out |= {x + k: (n, W) for k, n in sizes.items()}
            out |= {x + k + ".norm": (n if par else a.dim,) for k, n in sizes.items() if k != "v"}
            out |= {x + k + ".conv": (n, a.conv) for k, n in sizes.items() if a.conv}
            out |= {x + "sink": (a.heads,), x + "o": (W, a.heads * a.vdim)}
            if par:
                n, y = s.mixer.width, p + "mix.right."
                out |= {y + k: (n, W) for k in "zxg"} | {y + "z.b": (n,), y + "x.b": (n,), y + "o": (W, n)}
                out |= {p + "mix.left.out": (W,), p + "mix.right.out": (W,)}
            y = p + "mlp."
            if isinstance(f, DenseSpec):
                out |= {y + "up": (f.ff, W), y + "down": (W, f.ff)}
            elif f is not None:
                n = f.experts + f.identity
                out |= {y + "router": (n, W), y + "correction": (n,)}
                for e in range(f.experts):
                    out |= {f"{y}e{e}.gate": (f.ff, W), f"{y}e{e}.up": (f.ff, W), f"{y}e{e}.down": (W, f.ff)}
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
            if kind.startswith("norm") or kind == "out":
                return t.fill_(0.3 if kind.endswith("b") else 1.0)
            if kind in ("b", "sink", "correction", "conv"):
                return t.normal_(0.0, 0.1 if kind == "correction" else 0.5, generator=gen)
            return t.normal_(0.0, 1.0 if name == "embed" else std, generator=gen).to(torch.bfloat16)
        return cls._build(cfg, get, dev, tp_rank, tp_size, dtype)

    @classmethod
    def _build(cls, cfg, get, device, tp_rank, tp_size, dtype):
        w = cls(cfg, device, tp_rank, tp_size, dtype)

        def mat(t):
            return t.to(device=w.device, dtype=w.dtype)

        def vec(t):
            return t.to(device=w.device, dtype=torch.float32).contiguous().view(-1)

        def rows(t):
            return t.view(tp_size, t.shape[0] // tp_size, *t.shape[1:])[tp_rank]

        def cols(t):
            return t.view(t.shape[0], tp_size, t.shape[1] // tp_size)[:, tp_rank].contiguous()

        for i, s in enumerate(cfg.specs):
            a, f, p = s.attn, s.mlp, f"l{i}."
            par = isinstance(s.mixer, ParallelSpec)
            x, tp = p + ("mix.left." if par else "mix."), 1 if par else tp_size
            cut, cut_o = (rows, cols) if tp > 1 else (lambda t: t, lambda t: t)
            names = "q" if a.kv_from is not None else "qkv"
            conv = torch.cat([get(f"{x}{k}.conv") for k in names]).t().float().contiguous().to(w.device) if a.conv else None
            heads = A.Heads(a.heads // tp, a.kv_heads // tp, a.dim, a.vdim, a.scale, a.mask, cfg.norm_eps, vec(get(x + "q.norm")),
                            vec(get(x + "k.norm")) if len(names) > 1 else None, not par, vec(cut(get(x + "sink"))),
                            A.rope_freq(a.rot, a.base, w.device), conv, len(names) == 1)
            lw = {"heads": heads, "norm1": vec(get(p + "norm1")), "norm1b": vec(get(p + "norm1b")),
                  "o": Projection(mat(cut_o(get(x + "o"))))}
            parts = [(mat(torch.cat([cut(get(x + k)) for k in names])), 0)]
            if par:
                y = p + "mix.right."
                parts.append((mat(torch.cat([rows(get(y + k)) for k in "zxg"])), 0))
                lw["gru"] = R.Gru(vec(rows(get(y + "z.b"))), vec(rows(get(y + "x.b"))))
                lw["o2"] = Projection(mat(cols(get(y + "o"))))
                lw["out1"], lw["out2"] = vec(get(p + "mix.left.out")), vec(get(p + "mix.right.out"))
            lw["in"] = JointProjection(parts)
            if f is not None:
                lw["norm2"], lw["norm2b"] = vec(get(p + "norm2")), vec(get(p + "norm2b"))
            y = p + "mlp."
            if isinstance(f, DenseSpec):
                lw["up"], lw["down"] = Projection(mat(rows(get(y + "up")))), Projection(mat(cols(get(y + "down"))))
            elif f is not None:
                lw["gate"] = JointProjection([(mat(get(y + "router")), 0)])
                lw["router"] = M.Router(f.experts + f.identity, f.top, 1, 1, 1.0, vec(get(y + "correction")), softmax=True, renorm=False)
                ex = [[mat(c(get(f"{y}e{e}.{k}"))) for e in range(f.experts)]
                      for k, c in (("gate", rows), ("up", rows), ("down", cols))]
                lw["experts"] = M.ExpertWeights(*(torch.stack(t) for t in ex))
                lw["glu"] = M.Glu(f.limit, GLU_ALPHA, GLU_SHIFT)
            w.layers.append(lw)
        w.embed = mat(get("embed")).contiguous()
        w.head = Projection(mat(rows(get("head"))))
        w.final_norm = vec(get("final.norm"))
        if w.device.type == "cuda":
            torch.cuda.empty_cache()
        return w

    def nbytes(self) -> int:
        n = self.embed.numel() * self.embed.element_size() + self.head.nbytes()
        return n + sum(lw[k].nbytes() for lw in self.layers for k in ("in", "o", "o2", "up", "down", "gate", "experts") if k in lw)


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


class PemolornModel:
    """Stateless forward functions over :class:`PemolornWeights` + a :class:`GroupedCache`."""

    @staticmethod
    def kernel_sources(cfg, dtype) -> tuple:
        """csrc/kernels sources a run of this configuration launches kernels from."""
        src = {"elementwise", "stream", "branch", "qkv", "gqa"}
        for s in cfg.specs:
            if isinstance(s.mixer, ParallelSpec):
                src.add("gru")
            if isinstance(s.mlp, MoeSpec):
                src.add("moe")
        if dtype == torch.bfloat16:
            src |= {"gemm", "dgemm", "pgemm"}
        return tuple(sorted(src))

    def __init__(self, weights: PemolornWeights, tp_group=None, custom_ar=None):
        self.w = weights
        self.cfg = weights.cfg
        self.tp_group = tp_group
        self.custom_ar = custom_ar

    # ---------------------------------------------------------------- engine interface
    def new_cache(self, num_blocks: int, dtype=None, device=None, sequences: int | None = None) -> GroupedCache:
        if dtype not in (None, self.w.dtype):
            raise ValueError(f"cache in the model's dtype ({self.w.dtype}), not {dtype}")
        layers = []
        for s, lw in zip(self.cfg.specs, self.w.layers):
            a, pool = lw["heads"], s.attn.mask.pool
            own = (a.G, a.D, pool, A.pool_entries(pool) if pool else 0)
            layers.append({"heads": own if s.attn.kv_from is None else s.attn.kv_from,
                           "tail": (a.taps - 1, a.columns) if a.taps > 1 else None,
                           "recur": lw["gru"].width if "gru" in lw else None})
        return GroupedCache(layers, num_blocks, sequences or min(num_blocks, DEFAULT_SEQUENCES), device or self.w.device, self.w.dtype)

    def decode_partitions(self, B: int, max_blocks: int) -> int:
        """Key slices per sequence of a B-row decode step over block tables ``max_blocks`` wide."""
        ctx = max_blocks * KV_BLOCK
        return max(A.decode_slices(B, a.H, a.G, a.D, a.mask.visible(ctx), self.w.dtype) for a in (lw["heads"] for lw in self.w.layers))

    def decode_workspace(self, B: int, P: int) -> int:
        return max(B * lw["heads"].H * P * (lw["heads"].D + 2) for lw in self.w.layers) if P > 1 else 1

    def _tiles(self, a: A.Heads) -> str:
        return f"tiles_{a.H}_{a.G}_{A.prompt_rows(self.w.dtype, a.D)}"

    def plan_prefill(self, cu, ctx, slots, states) -> dict:
        """Host-side launch plan of a packed pass over portions cu / ctx in state slots ``states``: int32 arrays for
        the device."""
        n = np.diff(np.asarray(cu))
        plan = {"states": np.asarray(states, np.int32), "row_states": np.repeat(np.asarray(states, np.int32), n),
                "lead": np.concatenate([np.arange(k, dtype=np.int32) for k in n])}
        for s, lw in zip(self.cfg.specs, self.w.layers):
            a = lw["heads"]
            if self._tiles(a) not in plan:
                plan[self._tiles(a)] = A.prompt_tiles(cu, ctx, a.H, a.G, A.prompt_rows(self.w.dtype, a.D))
            if a.mask.pool and f"ended_{a.mask.pool}" not in plan:
                plan[f"ended_{a.mask.pool}"] = A.ended_blocks(cu, ctx, a.mask.pool)
            if "gru" in lw and "chunks" not in plan:
                plan["chunks"], plan["chunk_cu"] = R.chunk_plan(cu)
        return plan

    # ---------------------------------------------------------------- forward
    def forward_prefill(self, ids, positions, slots, cu_q, ctx_lens, block_tables, kv, last_idx=None, plan=None):
        """Packed portions of prompts (down to one token each), their launch plan from :meth:`plan_prefill`.  Returns
        the final-normed hidden states of rows ``last_idx`` (or all rows)."""
        h = self._layers(ids, _Pass(positions, slots, plan["states"], ctx_lens, block_tables, kv, plan, cu_q))
        return h if last_idx is None else h.index_select(0, last_idx)

    def forward_decode(self, ids, positions, slots, ctx_lens, block_tables, kv, attn_workspace=None, part_blocks=-1,
                       shared_blocks=None, states=None):
        """One token per sequence, ``states`` their state slots.  Returns the final-normed hidden states [B, W].
        ``part_blocks``: -P, P key slices per sequence (the engine's form); ``shared_blocks`` is not used."""
        return self._layers(ids, _Pass(positions, slots, states, ctx_lens, block_tables, kv, P=max(1, -part_blocks),
                                       workspace=attn_workspace))

    def _layers(self, ids, io: _Pass) -> torch.Tensor:
        W, dt, eps = self.cfg.hidden, self.w.dtype, self.cfg.norm_eps
        x = S.embed_f32(self.w.embed, ids, torch.empty(ids.numel(), W, dtype=torch.float32, device=ids.device))
        h = torch.empty(ids.numel(), W, dtype=dt, device=ids.device)
        gains = [g for lw in self.w.layers for g in ((lw["norm1"], lw["norm2"]) if "norm2" in lw else (lw["norm1"],))]
        gains = iter(gains + [self.w.final_norm])
        N.branch_norm(x, None, next(gains), eps, h)
        for i, lw in enumerate(self.w.layers):
            N.branch_norm(x, self._mixer(i, h, io), next(gains), eps, h)
            if "norm2" in lw:
                N.branch_norm(x, self._feed(i, h), next(gains), eps, h)
        return h

    def _mixer(self, i, h, io: _Pass) -> N.Branch:
        lw = self.w.layers[i]
        decode, hs = io.plan is None, h[None]
        c = lw["in"].joint(hs) if decode else [lw["in"].act(j, hs) for j in range(len(lw["in"].sizes))]
        b = N.Branch(lw["norm1b"], self.cfg.norm_eps)
        s = None
        if "gru" in lw:
            s = self._recur(i, c[1], io)
        o = self._attend(i, c[0], io)
        if s is None:
            b.y = self._sum(lw["o"].slabs(o))
        else:
            b.y, b.w, b.w2 = lw["o"].slabs(o, own=True), lw["out1"], lw["out2"]
            b.y2 = self._sum(lw["o2"].slabs(s))
        return b

    def _attend(self, i, cols: Cols, io: _Pass) -> torch.Tensor:
        """Attention of layer i: its heads' outputs [T, H vdim]."""
        a, rows, tail = self.w.layers[i]["heads"], io.kv.heads[i], io.kv.tail[i]
        if io.plan is None:
            q = A.qkv_rows(a, cols, rows, io.positions, io.slots, io.states, io.block_tables, tail)
            return A.attention(a, q, rows, io.block_tables, io.ctx_lens, P=io.P, workspace=io.workspace)
        p = io.plan
        q = A.qkv_rows(a, cols, rows, io.positions, io.slots, p["row_states"], io.block_tables, tail, p["lead"])
        A.conv_tail(a, cols, io.cu_q, io.ctx_lens, io.states, tail)
        if a.mask.pool:
            A.pool_rows(a, rows, p[f"ended_{a.mask.pool}"], io.block_tables)
        return A.attention(a, q, rows, io.block_tables, io.ctx_lens, io.cu_q, p[self._tiles(a)])

    def _recur(self, i, cols: Cols, io: _Pass) -> torch.Tensor:
        """Recurrence of layer i: its gated states [T, width]."""
        g, state = self.w.layers[i]["gru"], io.kv.recur[i]
        n = g.width
        zxg = [Cols(cols.t, cols.c0 + k * n, n) for k in range(3)]
        out = torch.empty(cols.rows, n, dtype=self.w.dtype, device=cols.t.device)
        if io.plan is None:
            return R.step(g, *zxg, io.states, io.ctx_lens, state, out)
        return R.prefill(g, *zxg, io.states, io.cu_q, io.ctx_lens, io.plan["chunks"], io.plan["chunk_cu"], state, out)

    def _sum(self, slabs) -> torch.Tensor:
        """A sharded product's slabs as one all-reduced slab (TP), else as they are."""
        if self.w.tp_size == 1:
            return slabs
        part = slabs[:1].clone()
        for p in slabs[1:]:                # elementwise adds: nothing a captured graph could not hold
            part.add_(p)
        torch.distributed.all_reduce(part, group=self.tp_group)
        return part

    def _feed(self, i, h) -> N.Branch:
        """Layer i's feed-forward of h as the branch it adds."""
        lw, f = self.w.layers[i], self.cfg.specs[i].mlp
        b = N.Branch(lw["norm2b"], self.cfg.norm_eps)
        if isinstance(f, DenseSpec):
            b.y = self._sum(lw["down"].slabs(lw["up"].relu_sq(h)))
            return b
        ids, wt = M.route(lw["gate"].slabs(0, h[None]), lw["router"])
        rows, pos = M.experts(h, lw["experts"], ids, lw["glu"])
        if self.w.tp_size == 1:
            b.routed = (rows, pos, wt, ids, f.experts, h)
            return b
        own = (ids >= f.experts)[..., None]
        y = self._sum((rows[pos.long()].float() * wt[..., None]).masked_fill(own, 0.0).sum(1)[None])
        b.y = y.add_((wt[..., None] * own).sum(1) * h.float())
        return b

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
