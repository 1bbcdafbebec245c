"""Zisapel decoder: layers of two kinds -- a linear recurrence with data-dependent decays, and sliding-window
latent attention with rotary positions and sinks -- each with a dense or a routed feed-forward or none; every
sublayer reads the unnormed stream, its result is gated, layer-normed and added.

MI355X layout choices:
  * a sequence's state is a slot of fixed size (fp32 recurrent state, the layers' input rows of its last two
    tokens); attention layers cache one row per token, latent and shared rotated key part side by side, and
    attend in the latent space (ops.latent);
  * everything a layer multiplies its inputs with is ONE packed matrix over several inputs (the row itself, the
    shifted row or its mixes): a decode step takes it in one launch whose fp32 slabs the next kernel sums, a
    prompt takes each part on the prefill product;
  * a branch's slab sum, gate, layer norm, residual sum and (decode) the next layer's token shift are one kernel
    (ops.gated); prompt portions of the recurrence run chunk-parallel on fp32 matrix cores (ops.wkv);
  * experts are routed and sorted on the device, so the decode step is one captured graph (ops.moe);
  * tensor parallel: heads, feed-forward columns (each expert's too) and vocabulary are sharded, gates and
    latents replicated; one all-reduce per sublayer.

Activations and weights are bf16, or fp32 throughout (``dtype=torch.float32``: library products and the fp32
forms of the same kernels).
"""
from __future__ import annotations

import dataclasses
import math

import numpy as np
import torch

from ..ops import gated as G
from ..ops import kernels as K
from ..ops import latent as L
from ..ops import moe as M
from ..ops import stream as S
from ..ops import wkv as R
from ..ops.reference import KV_BLOCK, interleave_gate_up, row_meta
from ..runtime.kv_cache import HybridCache
from .checkpoint import open_tensors, tensor_reader
from .decoder import argmax_keys
from .projection import JointProjection, Projection

GLU_ALPHA = 1.702     # slope of the gate's sigmoid
GLU_SHIFT = 1.0       # added to the clamped up projection
MIXES = "rkvgw"       # inputs of the recurrence's projections
DEFAULT_SEQUENCES = 256


@dataclasses.dataclass(frozen=True)
class WkvSpec:
    """Recurrence of one layer; ``rank`` of the decays' low-rank product."""
    heads: int
    dim: int
    rank: int


@dataclasses.dataclass(frozen=True)
class WindowSpec:
    """Latent attention of one layer; ``scaling`` of the rotary frequencies as sorted items."""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    window: int
    base: float
    scaling: tuple | None


@dataclasses.dataclass(frozen=True)
class GluSpec:
    """Clamped GLU feed-forward."""
    ff: int
    limit: float


@dataclasses.dataclass(frozen=True)
class MoeSpec:
    """Routed experts, with a shared one (``shared`` its inner size) or without."""
    ff: int
    experts: int
    top: int
    groups: int
    keep: int
    scale: float
    shared: int | None


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: WkvSpec | WindowSpec
    mlp: GluSpec | MoeSpec | None


@dataclasses.dataclass(frozen=True)
class ZisapelConfig:
    name: str
    vocab_size: int
    hidden: int
    specs: tuple[LayerSpec, ...]
    norm_eps: float
    logit_scale: float
    # nothing in the design bounds a sequence; the cache pool does
    max_positions: int = 1 << 20
    # the design names no special tokens: -1 never matches a generated one
    bos_id: int = 1
    eos_id: int = -1

    @property
    def layers(self) -> int:
        return len(self.specs)

    def num_params(self) -> int:
        return sum(math.prod(s) for s in ZisapelWeights.tensor_shapes(self).values())

    def flops_per_token(self, ctx: int = 0) -> float:
        """Product flops per token (chosen experts only; + latent attention over the visible part of ``ctx`` keys)."""
        W = self.hidden
        f = 2.0 * W * self.vocab_size
        for s in self.specs:
            m, p = s.mixer, s.mlp
            f += 2 * W * W * (2 if p is not None else 1)
            if isinstance(m, WkvSpec):
                f += 2 * m.heads * m.dim * (5 * W + m.rank) + 2 * W * m.rank + 6 * m.heads * m.dim ** 2
            else:
                f += 2 * W * (m.heads * (m.dim + m.rot_dim + 2 * m.vdim) + m.kv_rank + m.rot_dim)
                f += 2 * m.heads * m.kv_rank * (m.dim + m.vdim)
                f += 2 * m.heads * (2 * m.kv_rank + m.rot_dim) * (min(ctx, m.window) if m.window else ctx)
            if isinstance(p, GluSpec):
                f += 6 * W * p.ff
            elif p is not None:
                f += 6 * W * (p.ff * p.top + (p.shared or 0)) + 2 * W * p.experts
        return f


def config_from_json(c: dict, name: str = "zisapel", ckpt_dir=None) -> ZisapelConfig:
    """ZisapelConfig from a parsed config.json and (``ckpt_dir``) the shapes of the tensors beside it."""
    tensors, specs = None, []
    for i, layer in enumerate(c["layers"]):
        m, f, kind = layer["mixer"], layer.get("mlp"), layer["type"]
        if kind == "wkv":
            rank = m.get("rank")
            if rank is None and ckpt_dir is not None:
                tensors = tensors or open_tensors(ckpt_dir)
                rank = tensors[f"l{i}.mix.w1"].get_slice(f"l{i}.mix.w1").get_shape()[0]
            if rank is None:
                raise ValueError(f"layer {i}: the rank of the decay product is not in config.json: give the tensors' folder")
            mixer = WkvSpec(int(m["heads"]), int(m["dim"]), int(rank))
        elif kind == "latent_attention":
            rot, mask = m["rot"], m.get("mask") or {}
            if int(rot["dims"]) != int(m["rot_dim"]):
                raise NotImplementedError(f"layer {i}: rot.dims {rot['dims']} differs from rot_dim {m['rot_dim']}")
            sc = rot.get("scaling")
            mixer = WindowSpec(int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"]),
                               float(m["scale"]), int(mask.get("size") or 0), float(rot["base"]),
                               tuple(sorted((k, float(v)) for k, v in sc.items())) if sc else None)
        else:
            raise NotImplementedError(f"layer {i}: mixer {kind!r} (Zisapel has wkv and latent_attention)")
        if f is None:
            mlp = None
        elif f["kind"] == "dense":
            mlp = GluSpec(int(f["ff"]), float(f["limit"]))
        elif f["kind"] == "moe":
            r, sh = f["router"], f.get("shared")
            g = r.get("groups") or {"count": 1, "keep": 1}
            mlp = MoeSpec(int(f["expert"]["ff"]), int(r["experts"]), int(r["top"]), int(g["count"]), int(g["keep"]),
                          float(r["scale"]), int(sh["ff"]) if sh else None)
        else:
            raise NotImplementedError(f"layer {i}: feed-forward {f['kind']!r} (Zisapel has dense and moe)")
        specs.append(LayerSpec(mixer, mlp))
    return ZisapelConfig(name, int(c["vocab"]), int(c["width"]), tuple(specs), float(c["norm"]["eps"]), float(c["logit_scale"]))


def pattern_config(name: str, vocab: int, hidden: int, layers: int, wkv: WkvSpec, window: WindowSpec, dense: GluSpec,
                   moe: MoeSpec, eps: float = 1e-6, logit_scale: float = 1.0, max_positions: int = 1 << 20) -> ZisapelConfig:
    """Layers of the design's pattern: three recurrent ones to one that attends, dense and routed in turn."""
    cycle = (LayerSpec(wkv, dense), LayerSpec(window, moe), LayerSpec(wkv, dense), LayerSpec(wkv, moe))
    return ZisapelConfig(name, vocab, hidden, tuple(cycle[i % 4] for i in range(layers)), eps, logit_scale, max_positions)


_YARN = (("factor", 8.0), ("fast", 32.0), ("original", 4096.0), ("slow", 1.0))
PRESETS: dict[str, ZisapelConfig] = {
    # Mistral-7B's width, depth, attention heads and dense feed-forward
    "zisapel-7b": pattern_config("zisapel-7b", 32000, 4096, 32, WkvSpec(64, 64, 64),
                                 WindowSpec(32, 128, 64, 128, 512, 192 ** -0.5, 2048, 10000.0, _YARN), GluSpec(14336, 7.0),
                                 MoeSpec(1024, 32, 4, 4, 2, 2.5, 4096), max_positions=32768),
    "zisapel-small": pattern_config("zisapel-small", 32000, 1024, 4, WkvSpec(16, 64, 32),
                                    WindowSpec(8, 128, 64, 128, 256, 192 ** -0.5, 512, 10000.0, _YARN), GluSpec(2816, 7.0),
                                    MoeSpec(256, 16, 2, 4, 2, 2.0, 512), max_positions=8192),
    "tiny-zisapel": pattern_config("tiny-zisapel", 512, 128, 4, WkvSpec(4, 32, 16), WindowSpec(2, 48, 16, 32, 64, 0.2, 40, 5000.0, _YARN),
                                   GluSpec(192, 3.0), MoeSpec(64, 8, 2, 4, 2, 1.5, 64), logit_scale=0.5, max_positions=4096),
}


def get_config(name_or_cfg) -> ZisapelConfig:
    return name_or_cfg if isinstance(name_or_cfg, ZisapelConfig) else PRESETS[name_or_cfg]


class ZisapelWeights:
    """Per-rank (TP-sharded) weights on one device: matrices in ``dtype``, vectors in fp32."""

    def __init__(self, cfg: ZisapelConfig, device, tp_rank: int = 0, tp_size: int = 1, dtype=torch.bfloat16):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"Zisapel weights in bfloat16 or float32, not {dtype}")
        sharded = [cfg.vocab_size]
        for s in cfg.specs:
            sharded.append(s.mixer.heads)
            if s.mlp is not None:
                sharded += [s.mlp.ff, getattr(s.mlp, "shared", None) or 0]
        if any(n % tp_size for n in sharded):
            raise ValueError(f"{cfg.name}: heads / ff / vocab must divide tp_size={tp_size}")
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.tp_rank, self.tp_size = tp_rank, tp_size
        self.vocab_shard = cfg.vocab_size // tp_size
        self.layers: list[dict] = []
        self.embed = self.head = self.final_norm = None

    @staticmethod
    def tensor_shapes(cfg: ZisapelConfig) -> dict[str, tuple]:
        """Every tensor of a checkpoint and its shape."""
        W = cfg.hidden
        out = {"embed": (cfg.vocab_size, W), "head": (cfg.vocab_size, W), "final.norm": (W,)}
        for i, s in enumerate(cfg.specs):
            m, f, p = s.mixer, s.mlp, f"l{i}."
            out |= {p + "norm1": (W,), p + "shift": (W,), p + "rg1": (W, W), p + "rg1.b": (W,)}
            x = p + "mix."
            if isinstance(m, WkvSpec):
                HD = m.heads * m.dim
                out |= {x + "mu." + k: (W,) for k in MIXES}
                out |= {x + k: (HD, W) for k in "rkvg"}
                out |= {x + "w1": (m.rank, W), x + "w2": (HD, m.rank), x + "w0": (HD,), x + "u": (m.heads, m.dim),
                        x + "norm": (HD,), x + "o": (W, HD)}
            else:
                HV = m.heads * m.vdim
                out |= {x + "q": (m.heads * (m.dim + m.rot_dim), W), x + "dkv": (m.kv_rank + m.rot_dim, W),
                        x + "dkv.norm": (m.kv_rank,), x + "uk": (m.heads * m.dim, m.kv_rank), x + "uv": (HV, m.kv_rank),
                        x + "sink": (m.heads,), x + "g": (HV, W), x + "o": (W, HV)}
            if f is None:
                continue
            out |= {p + "norm2": (W,), p + "rg2": (W, W), p + "rg2.b": (W,)}

            def glu(at, ff):
                return {at + "gate": (ff, W), at + "up": (ff, W), at + "down": (W, ff)}
            y = p + "mlp."
            if isinstance(f, GluSpec):
                out |= glu(y, f.ff)
                continue
            out |= {y + "router": (f.experts, W), y + "correction": (f.experts,)}
            for e in range(f.experts):
                out |= glu(f"{y}e{e}.", f.ff)
            if f.shared:
                out |= glu(y + "shared.", f.shared)
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
            t = torch.empty(*shapes[name], dtype=torch.float32, device=dev)
            kind = name.rsplit(".", 1)[-1]
            if kind.startswith("norm"):
                return t.fill_(1.0 if not kind[4:] else 0.3)
            if kind == "shift" or ".mu." in name:
                return t.uniform_(0.0, 1.0, generator=gen)
            if kind == "w0":
                return t.uniform_(-6.0, 0.0, generator=gen)
            if kind in ("b", "u", "sink", "correction"):
                return t.normal_(0.0, 0.1 if kind == "correction" else 0.5, generator=gen)
            return t.normal_(0.0, 1.0 if name == "embed" else std, generator=gen).to(torch.bfloat16)
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

        def glu(at, ff):
            """Joint gate / up product (8-row interleaved where the size allows) and the down product."""
            gu = torch.cat([mat(rows(get(at + "gate"))), mat(rows(get(at + "up")))])
            inter = (ff // tp_size) % 8 == 0
            fused = inter and Projection.packs(gu, gu.shape[0], cfg.hidden)
            return {"gate_up": Projection(interleave_gate_up(gu) if inter else gu, swiglu=fused), "interleaved": inter,
                    "down": Projection(mat(cols(get(at + "down")))), "ff": ff // tp_size}

        for i, s in enumerate(cfg.specs):
            m, f, p, x = s.mixer, s.mlp, f"l{i}.", f"l{i}.mix."
            H = m.heads // tp_size
            lw = {"H": H, "norm1": vec(get(p + "norm1")), "shift": vec(get(p + "shift")), "rg1_b": vec(get(p + "rg1.b")),
                  "mus": None, "o": Projection(mat(cols(get(x + "o"))))}
            gate1 = (mat(get(p + "rg1")), 0)
            if isinstance(m, WkvSpec):
                lw["mus"] = torch.stack([vec(get(x + "mu." + k)) for k in MIXES])
                lw["in"] = JointProjection([gate1] + [(mat(rows(get(x + k))), 1 + j) for j, k in enumerate("rkvg")] +
                                           [(mat(get(x + "w1")), 1 + MIXES.index("w"))])
                lw["wkv"] = R.Wkv(H, m.dim, m.rank, rows(get(x + "w2")).to(w.device), vec(rows(get(x + "w0"))),
                                  vec(rows(get(x + "u"))), vec(rows(get(x + "norm"))), cfg.norm_eps)
            else:
                lw["in"] = JointProjection([gate1, (mat(rows(get(x + "q"))), 1), (mat(get(x + "dkv")), 1),
                                            (mat(rows(get(x + "g"))), 1)])
                lw["dkv_norm"], lw["sink"] = vec(get(x + "dkv.norm")), vec(rows(get(x + "sink")))
                # the unrotated query goes into the latent space: [H, rank, dim], rows up to the latent's stride
                uk = mat(rows(get(x + "uk"))).view(H, m.dim, m.kv_rank)
                lw["uk"] = L.HeadWeight(uk.transpose(1, 2), n_out=L.padded_rank(m.kv_rank))
                lw["uv"] = L.HeadWeight(mat(rows(get(x + "uv"))).view(H, m.vdim, m.kv_rank))
                if (m.dim == m.vdim == L.EXPANDED_DIM and m.rot_dim <= L.ROT_COLS and m.rot_dim % 8 == 0
                        and Projection.packs(uk, H * m.dim, m.kv_rank) and K.prefill_rows(H, H) == 256):
                    # long portions: keys and values per head from two products (ops.latent.expand)
                    lw["uk_full"] = K.pack_dgemm_weight(uk.reshape(H * m.dim, m.kv_rank).contiguous())
                    lw["uv_full"] = mat(rows(get(x + "uv"))).contiguous()
                lw["rope"] = L.yarn_rope(m.rot_dim, m.base, dict(m.scaling) if m.scaling else None, w.device)
            if f is not None:
                lw["norm2"], lw["rg2_b"] = vec(get(p + "norm2")), vec(get(p + "rg2.b"))
            if isinstance(f, GluSpec):
                lw["glu"], lw["limit"] = glu(p + "mlp.", f.ff), f.limit
                lw["ff_in"] = JointProjection([(mat(get(p + "rg2")), 0)])
            elif f is not None:
                y = p + "mlp."
                lw["ff_in"] = JointProjection([(mat(get(p + "rg2")), 0), (mat(get(y + "router")), 0)])
                lw["router"] = M.Router(f.experts, f.top, f.groups, f.keep, f.scale, vec(get(y + "correction")))
                ex = [[mat(cut(get(f"{y}e{e}.{k}"))) for e in range(f.experts)]
                      for k, cut in (("gate", rows), ("up", rows), ("down", cols))]
                lw["experts"] = M.ExpertWeights(*(torch.stack(t) for t in ex))
                lw["shared"] = glu(y + "shared.", f.shared) if f.shared else None
            w.layers.append(lw)
        w.embed = mat(get("embed")).contiguous()
        w.head = Projection(mat(rows(get("head"))))
        w.final_norm = vec(get("final.norm"))
        if w.device.type == "cuda":
            torch.cuda.empty_cache()
        return w

    def nbytes(self) -> int:
        n = self.embed.numel() * self.embed.element_size() + self.head.nbytes()
        for lw in self.layers:
            n += sum(lw[k].nbytes() for k in ("o", "in", "uk", "uv", "uk_full", "ff_in", "experts") if k in lw)
            n += lw["uv_full"].numel() * 2 if "uv_full" in lw else 0
            for k in ("glu", "shared"):
                if lw.get(k):
                    n += lw[k]["gate_up"].nbytes() + lw[k]["down"].nbytes()
        return n


class ZisapelModel:
    """Stateless forward functions over :class:`ZisapelWeights` + a :class:`HybridCache`."""

    @staticmethod
    def kernel_sources(cfg, dtype) -> tuple:
        """csrc/kernels sources a run of this configuration launches kernels from."""
        src = {"elementwise", "stream", "gated"}
        for s in cfg.specs:
            src.add("wkv" if isinstance(s.mixer, WkvSpec) else "latent")
            if isinstance(s.mlp, MoeSpec):
                src.add("moe")
            if dtype == torch.bfloat16 and isinstance(s.mixer, WindowSpec) and s.mixer.dim == s.mixer.vdim == L.EXPANDED_DIM:
                src.add("attention")
        if dtype == torch.bfloat16:
            src |= {"gemm", "dgemm", "pgemm"}
        return tuple(sorted(src))

    def __init__(self, weights: ZisapelWeights, tp_group=None, custom_ar=None):
        self.w = weights
        self.cfg = weights.cfg
        self.tp_group = tp_group
        self.custom_ar = custom_ar

    # ---------------------------------------------------------------- engine interface
    def new_cache(self, num_blocks: int, dtype=None, device=None, sequences: int | None = None) -> HybridCache:
        if dtype not in (None, self.w.dtype):
            raise ValueError(f"cache in the model's dtype ({self.w.dtype}), not {dtype}")
        ms = [(s.mixer, lw["H"]) for s, lw in zip(self.cfg.specs, self.w.layers)]
        return HybridCache([None if isinstance(m, WkvSpec) else self._cols(m)[0] for m, _ in ms],
                           [(H, m.dim, m.dim) if isinstance(m, WkvSpec) else None for m, H in ms], num_blocks,
                           sequences or min(num_blocks, DEFAULT_SEQUENCES), self.cfg.hidden, device or self.w.device, self.w.dtype)

    @staticmethod
    def _cols(m: WindowSpec) -> tuple[int, int]:
        """(columns of a cached row, of them the latent's)."""
        rv = L.padded_rank(m.kv_rank)
        return rv + L.padded_rank(m.rot_dim), rv

    def _windows(self):
        """(layer, mixer, heads here, row columns, value columns) of every layer that attends."""
        for i, s in enumerate(self.cfg.specs):
            if isinstance(s.mixer, WindowSpec):
                yield i, s.mixer, self.w.layers[i]["H"], *self._cols(s.mixer)

    @staticmethod
    def _visible(m: WindowSpec, ctx: int) -> int:
        """Keys a decoded token's 64-key tiles cover."""
        return min(ctx, m.window + 63) if m.window else ctx

    def decode_partitions(self, B: int, max_blocks: int) -> int:
        """Key slices per sequence of a B-row decode step over block tables ``max_blocks`` wide."""
        best = 1
        for _, m, H, rs, _ in self._windows():
            ctx = self._visible(m, max_blocks * KV_BLOCK)
            best = max(best, L.decode_plan(B, H, rs, ctx)[1] if self.w.dtype == torch.bfloat16
                       else max(1, min(math.ceil(512 / B), ctx // 256)))
        return min(best, L.MAX_PARTITIONS)

    def decode_workspace(self, B: int, P: int) -> int:
        return max([1] + [B * H * P * (rv + 2) for _, _, H, _, rv in self._windows()]) if P > 1 else 1

    def _rows(self, i: int, decode: tuple | None = None) -> int:
        """Rows per attention work item of layer i; ``decode``: (B, key slices, context bound) of a decode step."""
        m, H = self.cfg.specs[i].mixer, self.w.layers[i]["H"]
        rs, rv = self._cols(m)
        plan = L.decode_plan(decode[0], H, rs, self._visible(m, decode[2]), decode[1]) if decode else None
        return L.rows_per_tile(self.w.dtype, rs, plan, rv)

    def plan_prefill(self, cu, ctx, slots, states) -> dict:
        """Host-side launch plan of a packed pass over portions cu / ctx in state slots ``states``: int32 arrays for
        the device."""
        chunks, chunk_cu = R.chunk_plan(cu)
        plan = {"states": np.asarray(states, np.int32), "chunks": chunks, "chunk_cu": chunk_cu,
                "meta": row_meta([(b - a, s) for a, b, s in zip(cu, cu[1:], states)]), "max_ctx": max(ctx)}
        for i, m, H, _, _ in self._windows():
            key = f"attn_{H}_{self._rows(i)}_{m.window}"
            if key not in plan:
                plan[key] = np.asarray(L.attn_tiles(cu, H, self._rows(i), ctx, m.window), np.int32).reshape(2, -1)
        for i, m, _, _, rv in self._windows():
            key = f"expand_{rv}_{m.window}"
            if "uk_full" in self.w.layers[i] and key not in plan:
                plan[key] = self._expand_pays(cu, ctx, rv, m.window)
                if plan[key] and f"gather_{m.window}" not in plan:
                    starts = [self._first_key(c - (b - a), m.window) for a, b, c in zip(cu, cu[1:], ctx)]
                    gt, base = L.gather_tiles(ctx, starts)
                    plan[f"gather_{m.window}"], plan[f"base_{m.window}"] = np.asarray(gt, np.int32), np.asarray(base, np.int32)
                    plan["pf_tiles"] = np.asarray(K.prefill_tiles(cu, 256, ctx), np.int32)
        return plan

    @staticmethod
    def _first_key(pos: int, window: int) -> int:
        return max(0, pos - window + 1) if window else 0

    @staticmethod
    def _expand_pays(cu, ctx, rv, window) -> bool:
        """Whether per-head keys and values of what the pass can see take less time than attention in the latent space
        with its two per-head products: flops per head (halved) over the rates measured on one MI355X."""
        d, latent, dense = 2 * L.EXPANDED_DIM, 0.0, 0.0
        for a, b, c in zip(cu, cu[1:], ctx):
            n, pos = b - a, c - (b - a)
            full = max(0, min(n, c - window)) if window else 0          # rows that see a whole window
            pairs = full * window + (n - full) * (pos + (n - full + 1) / 2)
            latent += pairs * (2 * rv + L.ROT_COLS) / 0.22 + n * rv * d / 0.14
            dense += pairs * (d + L.ROT_COLS) / 0.6 + (c - ZisapelModel._first_key(pos, window) + 32) * rv * d / 0.7
        return dense < latent

    # ---------------------------------------------------------------- forward
    def forward_prefill(self, ids, positions, slots, cu_q, ctx_lens, block_tables, kv, last_idx=None, plan=None):
        """Packed portions of prompts (down to one token each), their launch plan from :meth:`plan_prefill`.  Returns
        the final-normed hidden states of rows ``last_idx`` (or all rows)."""
        T, dt, dev = ids.numel(), self.w.dtype, ids.device
        x = S.embed_f32(self.w.embed, ids, torch.empty(T, self.cfg.hidden, dtype=torch.float32, device=dev))
        h = torch.empty(T, self.cfg.hidden, dtype=dt, device=dev)
        bufs: dict = {}
        for i, (s, lw) in enumerate(zip(self.cfg.specs, self.w.layers)):
            sh, part = self._shift(i, kv), lw["in"]
            acts = self._acts(sh, T, bufs)
            G.shift_mix(x, sh, plan["meta"], positions, acts)
            gate = part.act(0, acts)
            if isinstance(s.mixer, WkvSpec):
                o = torch.empty(T, lw["H"] * s.mixer.dim, dtype=dt, device=dev)
                R.prefill(lw["wkv"], *(part.act(j, acts) for j in (1, 2, 3, 4)), part.slabs(5, acts), plan["states"], cu_q,
                          ctx_lens, plan["chunks"], plan["chunk_cu"], kv.recur[i], o)
            else:
                rows = self._rows(i)
                tiles = plan[f"attn_{lw['H']}_{rows}_{s.mixer.window}"]
                keys = self._visible(s.mixer, plan["max_ctx"])
                o = self._attend(i, part.act(1, acts), part.slabs(2, acts), part.act(3, acts), positions, slots, ctx_lens,
                                 block_tables, kv, dict(cu_q=cu_q, tiles=(tiles[0], tiles[1]), rows=rows,
                                                        P=L.partitions(tiles.shape[1], keys)), plan)
            b = G.Branch(gate, lw["rg1_b"], lw["norm1"], self.cfg.norm_eps, y=self._sum(lw["o"].slabs(o)))
            G.gated_norm(x, b, dt, h if s.mlp is not None else None, kv.prev[i], plan["meta"], positions)
            if s.mlp is not None:
                ff, hs = lw["ff_in"], h[None]
                G.gated_norm(x, self._feed(i, h, ff.act(0, hs), ff.slabs(1, hs) if len(ff.sizes) > 1 else None), dt)
        return G.final_norm(x, self.w.final_norm, self.cfg.norm_eps, dt, None if last_idx is None else last_idx.to(torch.int32))

    def forward_decode(self, ids, positions, slots, ctx_lens, block_tables, kv, attn_workspace=None, part_blocks=-1,
                       shared_blocks=None, states=None):
        """One token per sequence, ``states`` their state slots.  Returns the final-normed hidden states [B, W].
        ``part_blocks``: -P, P key slices per sequence (the engine's form); ``shared_blocks`` is not used."""
        B, dt, dev, P = ids.numel(), self.w.dtype, ids.device, max(1, -part_blocks)
        x = S.embed_f32(self.w.embed, ids, torch.empty(B, self.cfg.hidden, dtype=torch.float32, device=dev))
        h = torch.empty(B, self.cfg.hidden, dtype=dt, device=dev)
        bufs: dict = {}

        def shift(b, j, h=None):
            """Add branch ``b`` to the stream and run layer j's token shift (past the last layer: none)."""
            if j >= self.cfg.layers:
                G.gated_shift(x, b, dt, h)
                return None
            sh = self._shift(j, kv)
            acts = self._acts(sh, B, bufs)
            G.gated_shift(x, b, dt, h, sh, positions, states, acts)
            return acts
        acts = shift(None, 0)
        for i, (s, lw) in enumerate(zip(self.cfg.specs, self.w.layers)):
            c = lw["in"].joint(acts)
            if isinstance(s.mixer, WkvSpec):
                o = torch.empty(B, lw["H"] * s.mixer.dim, dtype=dt, device=dev)
                R.step(lw["wkv"], *c[1:6], states, ctx_lens, kv.recur[i], o)
            else:
                o = self._attend(i, c[1], c[2], c[3], positions, slots, ctx_lens, block_tables, kv,
                                 dict(cu_q=None, rows=self._rows(i, (B, P, block_tables.shape[1] * KV_BLOCK)), P=P,
                                      workspace=attn_workspace))
            b = G.Branch(c[0], lw["rg1_b"], lw["norm1"], self.cfg.norm_eps, y=self._sum(lw["o"].slabs(o)))
            if s.mlp is None:
                acts = shift(b, i + 1)
            else:
                G.gated_shift(x, b, dt, h)
                acts = shift(self._feed(i, h, *lw["ff_in"].joint(h[None])), i + 1)
        return G.final_norm(x, self.w.final_norm, self.cfg.norm_eps, dt)

    def _shift(self, i, kv) -> G.Shift:
        lw = self.w.layers[i]
        return G.Shift(lw["shift"], lw["mus"], kv.prev[i])

    def _acts(self, sh, T, bufs) -> torch.Tensor:
        """The sublayer's input buffer, one per number of inputs and pass."""
        if sh.outputs not in bufs:
            bufs[sh.outputs] = sh.acts(T, self.w.dtype)
        return bufs[sh.outputs]

    def _sum(self, slabs) -> torch.Tensor:
        """A sharded product's slabs as one all-reduced slab (TP), else as they are."""
        if self.w.tp_size == 1:
            return slabs
        part = slabs[:1].clone()
        for p in slabs[1:]:                # elementwise adds: nothing a captured graph could not hold
            part.add_(p)
        torch.distributed.all_reduce(part, group=self.tp_group)
        return part

    def _attend(self, i, q, kv_cols, g, positions, slots, ctx_lens, block_tables, kv, attn, plan=None) -> torch.Tensor:
        """Latent attention of layer i: the gated heads [T, H vdim].  ``plan``: the launch plan of a packed pass."""
        lw, m = self.w.layers[i], self.cfg.specs[i].mixer
        T, H, dt, dev = q.rows, lw["H"], self.w.dtype, positions.device
        rs, rv = self._cols(m)

        def rope(qr):
            return L.latent_rope(kv_cols, m.kv_rank, lw["dkv_norm"], self.cfg.norm_eps, slots, kv.rows[i], q, H, m.dim,
                                 lw["rope"], positions, qr, m.vdim, g)
        if plan is not None and plan.get(f"expand_{rv}_{m.window}") and "uk_full" in lw:
            q2 = torch.empty(T, H, L.ROT_COLS, dtype=dt, device=dev)
            _, gate = rope(q2)
            k, vt, k2 = L.expand(kv.rows[i], block_tables, ctx_lens, plan[f"gather_{m.window}"], lw["uk_full"], lw["uv_full"], rv)
            return L.expanded_window_attention(q, q2, k, k2, vt, plan[f"base_{m.window}"], attn["cu_q"], ctx_lens, m.scale,
                                               plan["pf_tiles"], m.window, lw["sink"], gate,
                                               torch.empty(T, H * m.vdim, dtype=dt, device=dev))
        ql = torch.empty(T, H, rs, dtype=dt, device=dev)
        qn, gate = rope(ql[:, :, rv:])
        L.head_linear(qn, lw["uk"], ql)
        ol = L.latent_attention(ql, kv.rows[i], block_tables, ctx_lens=ctx_lens, scale=m.scale, window=m.window,
                                sink=lw["sink"], RV=rv, **attn)
        o = torch.empty(T, H, m.vdim, dtype=dt, device=dev)
        L.head_linear(ol, lw["uv"], o, gate)
        return o.view(T, H * m.vdim)

    def _glu(self, h, p, limit, alpha, beta, own=False) -> torch.Tensor:
        """fp32 slabs of a gated feed-forward's down product."""
        a = torch.empty(h.shape[0], p["ff"], dtype=h.dtype, device=h.device)
        if p["interleaved"]:
            p["gate_up"].glu(h, a, limit, alpha, beta)
        else:
            S.clamped_glu(p["gate_up"].slabs(h), a, limit, alpha, beta)
        return p["down"].slabs(a, own=own)

    def _feed(self, i, h, gate, router=None) -> G.Branch:
        """Layer i's feed-forward of h as the branch it adds; ``router``: the router's logits (routed layers)."""
        lw, f = self.w.layers[i], self.cfg.specs[i].mlp
        b = G.Branch(gate, lw["rg2_b"], lw["norm2"], self.cfg.norm_eps)
        if isinstance(f, GluSpec):
            b.y = self._sum(self._glu(h, lw["glu"], lw["limit"], GLU_ALPHA, GLU_SHIFT))
            return b
        ids, wt = M.route(router, lw["router"])
        rows, pos = M.experts(h, lw["experts"], ids)
        shared = self._glu(h, lw["shared"], M.INF, 1.0, 0.0) if lw["shared"] else None
        if self.w.tp_size == 1:
            b.y, b.routed = shared, (rows, pos, wt)
        else:
            y = (rows[pos.long()].float() * wt[..., None]).sum(1)[None]
            b.y = self._sum(torch.cat([y, shared]) if shared is not None else y)
        return b

    # ---------------------------------------------------------------- output
    def _local_logits(self, hidden):
        y = self.w.head.f32(hidden)
        return y if self.cfg.logit_scale == 1.0 else y.mul_(self.cfg.logit_scale)

    def logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """[B, V] fp32 logits (all-gathered over the vocabulary shards)."""
        local = self._local_logits(hidden)
        if self.w.tp_size == 1:
            return local
        parts = [torch.empty_like(local) for _ in range(self.w.tp_size)]
        torch.distributed.all_gather(parts, local, group=self.tp_group)
        return torch.cat(parts, -1)

    def greedy_ids(self, hidden: torch.Tensor, out: torch.Tensor) -> torch.Tensor:
        """Greedy next tokens into ``out``; under TP the shards' argmax keys are reduced instead of
        gathering the logits."""
        local = self._local_logits(hidden)
        if self.w.tp_size == 1:
            return K.sample(local, out, 0.0)
        keys = argmax_keys(local, self.w.tp_rank * self.w.vocab_shard)
        torch.distributed.all_reduce(keys, op=torch.distributed.ReduceOp.MAX, group=self.tp_group)
        out.copy_((0xFFFFFFFF - (keys & 0xFFFFFFFF)).to(torch.int32))
        return out

    def graph_collectives_ok(self, B: int) -> bool:
        return self.w.tp_size == 1
