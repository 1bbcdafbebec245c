"""Vofosun decoder: latent attention without positions, one norm per layer whose output both sublayers
read through a short causal convolution, their sum added at once, and a learned average over the results
of every earlier layer after each layer.

MI355X layout choices:
  * the cache holds the normed latents only (one row per token, shared by all heads) and attention runs
    in the latent space: W_uk is applied to the query and W_uv to the attention's output (ops.latent);
  * both down projections of a layer are one product, so are gate and up, and the attention's output
    projection and the feed-forward's down projection are ONE product over the concatenated
    [attention | feed-forward] activations -- the sublayers' sum comes out of the matrix cores in fp32;
  * the stream, its history over the layers, the norms and the convolution inputs are fp32; a prompt's
    rows take two kernels between layers (depth average + 1 / rms, convolution of both sublayers), a
    decoded row one (ops.stream);
  * tensor parallel: heads, feed-forward columns and vocabulary are sharded, the latents replicated; one
    all-reduce per layer (both sublayers' partials are already one sum).

Activations and weights are bf16, or fp32 throughout (``dtype=torch.float32``: library products and the
fp32 forms of the same kernels).
"""
from __future__ import annotations

import dataclasses
import math

import numpy as np
import torch

from ..ops import kernels as K
from ..ops import latent as L
from ..ops import stream as S
from ..ops.reference import KV_BLOCK, interleave_gate_up, tail_slots
from ..runtime.kv_cache import LatentKVCache
from .checkpoint import tensor_reader
from .decoder import argmax_keys
from .projection import Projection

GLU_ALPHA = 1.702     # slope of the gate's sigmoid
GLU_SHIFT = 1.0       # added to the clamped up projection
BIAS_COLS = 64        # input columns added for the gate / up biases on the packed path (one K step)


@dataclasses.dataclass(frozen=True)
class LatentSpec:
    """Latent attention of one layer."""
    heads: int
    dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float


@dataclasses.dataclass(frozen=True)
class GluSpec:
    """Clamped GLU feed-forward of one layer."""
    ff: int
    limit: float


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: LatentSpec
    mlp: GluSpec | None


@dataclasses.dataclass(frozen=True)
class VofosunConfig:
    name: str
    vocab_size: int
    hidden: int
    specs: tuple[LayerSpec, ...]
    norm_eps: float
    taps: int
    logit_softcap: float
    # nothing in the design bounds a sequence; the cache pool does
    max_positions: int = 1 << 20
    # the design names no special tokens: -1 never matches a generated one
    bos_id: int = 1
    eos_id: int = -1

    @property
    def layers(self) -> int:
        return len(self.specs)

    def num_params(self) -> int:
        n = 2 * self.vocab_size * self.hidden + self.hidden
        for i, s in enumerate(self.specs):
            m = s.mixer
            n += self.hidden * (m.q_rank + m.kv_rank + 1 + self.taps) + m.q_rank + m.kv_rank + i + 2
            n += m.heads * (m.dim * (m.q_rank + m.kv_rank) + m.vdim * (m.kv_rank + self.hidden))
            if s.mlp is not None:
                n += 3 * self.hidden * s.mlp.ff + 2 * s.mlp.ff + self.hidden * (1 + self.taps)
        return n

    def flops_per_token(self, ctx: int = 0) -> float:
        """Dense product flops per token (+ latent attention over ``ctx`` keys)."""
        f = 2.0 * self.hidden * self.vocab_size
        for s in self.specs:
            m = s.mixer
            f += 2 * self.hidden * (m.q_rank + m.kv_rank)
            f += 2 * m.heads * (m.dim * (m.q_rank + m.kv_rank) + m.vdim * (m.kv_rank + self.hidden))
            f += 4 * m.heads * m.kv_rank * ctx + (6 * self.hidden * s.mlp.ff if s.mlp is not None else 0)
        return f


def config_from_json(c: dict, name: str = "vofosun") -> VofosunConfig:
    """VofosunConfig from a parsed config.json."""
    specs = []
    for i, layer in enumerate(c["layers"]):
        if layer["type"] != "latent_attention":
            raise NotImplementedError(f"layer {i}: mixer {layer['type']!r} (Vofosun has latent_attention)")
        m, f = layer["mixer"], layer.get("mlp")
        if f is not None and f["kind"] != "dense":
            raise NotImplementedError(f"layer {i}: feed-forward {f['kind']!r} (Vofosun has dense)")
        specs.append(LayerSpec(
            LatentSpec(int(m["heads"]), int(m["dim"]), int(m["vdim"]), int(m["q_rank"]), int(m["kv_rank"]),
                       float(m["scale"])),
            GluSpec(int(f["ff"]), float(f["limit"])) if f is not None else None))
    return VofosunConfig(name, int(c["vocab"]), int(c["width"]), tuple(specs), float(c["norm"]["eps"]),
                         int(c["canon"]["taps"]), float(c["logit_softcap"]))


def uniform_config(name: str, vocab: int, hidden: int, layers: int, heads: int, dim: int, vdim: int, q_rank: int,
                   kv_rank: int, ff: int | None, taps: int = 4, limit: float = 7.0, eps: float = 1e-6,
                   softcap: float = 30.0, max_positions: int = 1 << 20) -> VofosunConfig:
    spec = LayerSpec(LatentSpec(heads, dim, vdim, q_rank, kv_rank, dim ** -0.5),
                     GluSpec(ff, limit) if ff is not None else None)
    return VofosunConfig(name, vocab, hidden, (spec,) * layers, eps, taps, softcap, max_positions)


PRESETS: dict[str, VofosunConfig] = {
    # Mistral-7B's width, depth, heads and feed-forward with the design's own attention
    "vofosun-7b": uniform_config("vofosun-7b", 32000, 4096, 32, 32, 128, 128, 1536, 512, 14336, max_positions=32768),
    "vofosun-small": uniform_config("vofosun-small", 32000, 1024, 4, 8, 128, 128, 384, 256, 2816, max_positions=8192),
    "tiny-vofosun": uniform_config("tiny-vofosun", 512, 192, 3, 4, 32, 48, 64, 96, 320, taps=3, max_positions=4096),
}


def get_config(name_or_cfg) -> VofosunConfig:
    return name_or_cfg if isinstance(name_or_cfg, VofosunConfig) else PRESETS[name_or_cfg]


class VofosunWeights:
    """Per-rank (TP-sharded) weights on one device: matrices in ``dtype``, vectors in fp32."""

    def __init__(self, cfg: VofosunConfig, device, tp_rank: int = 0, tp_size: int = 1, dtype=torch.bfloat16):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"Vofosun weights in bfloat16 or float32, not {dtype}")
        bad = cfg.vocab_size % tp_size or any(
            s.mixer.heads % tp_size or (s.mlp is not None and s.mlp.ff % tp_size) for s in cfg.specs)
        if bad:
            raise ValueError(f"{cfg.name}: heads / ff / vocab must divide tp_size={tp_size}")
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.tp_rank, self.tp_size = tp_rank, tp_size
        self.vocab_shard = cfg.vocab_size // tp_size
        self.layers: list[dict] = []
        self.embed = self.head = self.final_norm = None

    @staticmethod
    def tensor_shapes(cfg: VofosunConfig) -> dict[str, tuple]:
        """Every tensor of a checkpoint and its shape."""
        W = cfg.hidden
        out = {"embed": (cfg.vocab_size, W), "head": (cfg.vocab_size, W), "final.norm": (W,)}
        for i, s in enumerate(cfg.specs):
            m, p = s.mixer, f"l{i}."
            out |= {p + "norm1": (W,), p + "canon1": (W, cfg.taps), p + "dwa": (i + 2,),
                    p + "mix.dq": (m.q_rank, W), p + "mix.dq.norm": (m.q_rank,), p + "mix.uq": (m.heads * m.dim, m.q_rank),
                    p + "mix.dkv": (m.kv_rank, W), p + "mix.dkv.norm": (m.kv_rank,),
                    p + "mix.uk": (m.heads * m.dim, m.kv_rank), p + "mix.uv": (m.heads * m.vdim, m.kv_rank),
                    p + "mix.o": (W, m.heads * m.vdim)}
            if s.mlp is not None:
                F = s.mlp.ff
                out |= {p + "canon2": (W, cfg.taps), p + "mlp.gate": (F, W), p + "mlp.gate.b": (F,), p + "mlp.up": (F, W),
                        p + "mlp.up.b": (F,), p + "mlp.down": (W, F), p + "mlp.down.b": (W,)}
        return out

    @classmethod
    def from_safetensors(cls, cfg, ckpt_dir, device, tp_rank: int = 0, tp_size: int = 1, dtype=torch.bfloat16):
        get = tensor_reader(ckpt_dir, cls.tensor_shapes(cfg))
        return cls._build(cfg, get, device, tp_rank, tp_size, dtype)

    @classmethod
    def random(cls, cfg, device, seed: int = 0, tp_rank: int = 0, tp_size: int = 1, std: float = 0.02,
               dtype=torch.bfloat16):
        """Random weights of the full model, drawn tensor by tensor on the device (every TP rank draws the
        same full tensors and keeps its shard)."""
        dev = torch.device(device)
        gen = torch.Generator(device=dev)
        gen.manual_seed(seed * 1000003 + 77)
        shapes = cls.tensor_shapes(cfg)

        def get(name):
            s = shapes[name]
            t = torch.empty(*s, dtype=torch.float32, device=dev)
            kind = name.rsplit(".", 1)[-1]
            if name.endswith(("dq.norm", "dkv.norm")):
                return t.fill_(1.0)
            if kind == "dwa":
                t.normal_(0.0, 0.02, generator=gen)
                t[-1] += 1.0
                return t
            scale = 0.2 if kind.startswith("canon") else 1.0 if name == "embed" else std
            if name.endswith(("mix.o", "mlp.down")):
                scale /= math.sqrt(2 * cfg.layers)
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
            return t.view(t.shape[0], tp_size, t.shape[1] // tp_size)[:, tp_rank]

        for i, s in enumerate(cfg.specs):
            m, p = s.mixer, f"l{i}."
            H = m.heads // tp_size
            uk = mat(rows(get(p + "mix.uk"))).view(H, m.dim, m.kv_rank)
            uv = mat(rows(get(p + "mix.uv"))).view(H, m.vdim, m.kv_rank)
            out = [mat(cols(get(p + "mix.o")))]
            lw = {
                "H": H, "norm": 1.0 + vec(get(p + "norm1")), "convs": [vec(get(p + "canon1")).t().contiguous()], "dwa": vec(get(p + "dwa")),
                "down_in": Projection(torch.cat([mat(get(p + "mix.dq")), mat(get(p + "mix.dkv"))])),
                "dq_norm": vec(get(p + "mix.dq.norm")), "dkv_norm": vec(get(p + "mix.dkv.norm")),
                "uq": Projection(mat(rows(get(p + "mix.uq")))),
                # the query goes into the latent space: [H, rank, dim], rows up to the cache's stride
                "uk": L.HeadWeight(uk.transpose(1, 2), n_out=L.padded_rank(m.kv_rank)),
                "uv": L.HeadWeight(uv), "bias": None,
            }
            rs = L.padded_rank(m.kv_rank)
            if (m.dim == m.vdim == L.EXPANDED_DIM and rs == m.kv_rank and Projection.packs(uk, H * m.dim, rs)
                    and K.prefill_rows(H, H) == 256):
                # long portions: keys and values per head from two products (ops.latent.expand)
                lw["uk_full"] = K.pack_dgemm_weight(uk.reshape(H * m.dim, rs).contiguous())
                lw["uv_full"] = uv.reshape(H * m.vdim, rs).contiguous()
            if s.mlp is not None:
                gu = torch.cat([mat(rows(get(p + "mlp.gate"))), mat(rows(get(p + "mlp.up")))])
                lw["interleaved"] = (s.mlp.ff // tp_size) % 8 == 0
                gb, ub = rows(get(p + "mlp.gate.b")), rows(get(p + "mlp.up.b"))
                # packed: the biases are one more column of W (the input carries a constant 1 there), so
                # the product's epilogue has only the gate to do
                lw["fused_glu"] = lw["interleaved"] and Projection.packs(gu, gu.shape[0], cfg.hidden + BIAS_COLS)
                if lw["fused_glu"]:
                    pad = gu.new_zeros(gu.shape[0], BIAS_COLS)
                    pad[:, 0] = mat(torch.cat([gb, ub]))
                    gu = torch.cat([gu, pad], 1)
                else:
                    lw["gate_b"], lw["up_b"] = vec(gb), vec(ub)
                lw["gate_up"] = Projection(interleave_gate_up(gu) if lw["interleaved"] else gu, swiglu=lw["fused_glu"])
                lw["convs"].append(vec(get(p + "canon2")).t().contiguous())
                out.append(mat(cols(get(p + "mlp.down"))))
                lw["bias"] = vec(get(p + "mlp.down.b"))
            lw["out"] = Projection(torch.cat(out, 1))
            w.layers.append(lw)
        w.embed = mat(get("embed")).contiguous()
        w.head = Projection(mat(rows(get("head"))))
        w.final_norm = 1.0 + vec(get("final.norm"))
        if w.device.type == "cuda":
            torch.cuda.empty_cache()
        return w

    def nbytes(self) -> int:
        n = self.embed.numel() * self.embed.element_size() + self.head.nbytes()
        for lw in self.layers:
            n += sum(lw[k].nbytes() for k in ("down_in", "uq", "uk", "uv", "out"))
            n += lw["gate_up"].nbytes() if "gate_up" in lw else 0
            n += lw["uk_full"].nbytes() + lw["uv_full"].numel() * 2 if "uk_full" in lw else 0
        return n


class VofosunModel:
    """Stateless forward functions over :class:`VofosunWeights` + a :class:`LatentKVCache`."""

    @staticmethod
    def kernel_sources(cfg, dtype) -> tuple:
        """csrc/kernels sources a run of this configuration launches kernels from."""
        src = ("elementwise", "stream", "latent")
        if dtype == torch.bfloat16:
            src += ("gemm", "dgemm", "pgemm")
            if any(s.mixer.dim == s.mixer.vdim == L.EXPANDED_DIM for s in cfg.specs):
                src += ("attention",)
        return src

    def __init__(self, weights: VofosunWeights, tp_group=None, custom_ar=None):
        self.w = weights
        self.cfg = weights.cfg
        self.tp_group = tp_group
        self.custom_ar = custom_ar

    # ---------------------------------------------------------------- engine interface
    def new_cache(self, num_blocks: int, dtype=None, device=None, sequences: int | None = None) -> LatentKVCache:
        if dtype not in (None, self.w.dtype):
            raise ValueError(f"latent cache in the model's dtype ({self.w.dtype}), not {dtype}")
        return LatentKVCache([s.mixer.kv_rank for s in self.cfg.specs], num_blocks, self.cfg.hidden, tail_slots(self.cfg.taps),
                             device or self.w.device, self.w.dtype)

    def decode_partitions(self, B: int, max_blocks: int) -> int:
        """Key slices per sequence of a B-row decode step over block tables ``max_blocks`` wide."""
        if self.w.dtype != torch.bfloat16:
            return max(1, min(math.ceil(512 / B), max_blocks // 8))
        return max(L.decode_plan(B, lw["H"], self._rs(i), max_blocks * KV_BLOCK)[1] for i, lw in enumerate(self.w.layers))

    def decode_workspace(self, B: int, P: int) -> int:
        return max(B * lw["H"] * P * (self._rs(i) + 2) for i, lw in enumerate(self.w.layers)) if P > 1 else 1

    def _rs(self, i: int) -> int:
        return L.padded_rank(self.cfg.specs[i].mixer.kv_rank)

    def _rows(self, i: int, decode: tuple | None = None) -> int:
        """Rows per attention work item of layer i; ``decode``: (B, key slices, context bound) of a decode step."""
        rs, H = self._rs(i), self.w.layers[i]["H"]
        return L.rows_per_tile(self.w.dtype, rs, L.decode_plan(decode[0], H, rs, decode[2], decode[1]) if decode else None)

    def plan_prefill(self, cu, ctx, slots) -> dict:
        """Host-side launch plan of a packed pass over portions cu / ctx: int32 arrays for the device."""
        por = [(cu[s], cu[s + 1] - cu[s], ctx[s] - (cu[s + 1] - cu[s]), s) for s in range(len(ctx))]
        plan = {"conv_tiles": S.conv_tiles(por)}
        for i, lw in enumerate(self.w.layers):
            key = f"attn_{lw['H']}_{self._rows(i)}"
            if key not in plan:
                plan[key] = np.asarray(L.attn_tiles(cu, lw["H"], self._rows(i), ctx), np.int32).reshape(2, -1)
        plan["max_ctx"] = max(ctx)
        for i, lw in enumerate(self.w.layers):
            rs = self._rs(i)
            if "uk_full" in lw and f"expand_{rs}" not in plan:
                plan[f"expand_{rs}"] = self._expand_pays(cu, ctx, rs)
                if plan[f"expand_{rs}"] and "gather" not in plan:
                    gt, base = L.gather_tiles(ctx)
                    plan["gather"], plan["tok_base"] = np.asarray(gt, np.int32), np.asarray(base, np.int32)
                    plan["pf_tiles"] = np.asarray(K.prefill_tiles(cu, 256, ctx), np.int32)
        return plan

    @staticmethod
    def _expand_pays(cu, ctx, rs) -> bool:
        """Whether per-head keys and values of the pass's contexts cost fewer flops (per head, halved) than
        attention in the latent space with its two per-head products."""
        d, latent, dense = 2 * L.EXPANDED_DIM, 0.0, 0.0
        for s in range(len(ctx)):
            n = cu[s + 1] - cu[s]
            pairs = n * (ctx[s] - n / 2)
            latent += pairs * 2 * rs + n * rs * d
            dense += pairs * d + -(-ctx[s] // 64) * 64 * rs * d
        return dense < latent

    # ---------------------------------------------------------------- forward
    def forward_prefill(self, ids, positions, slots, cu_q, ctx_lens, block_tables, kv, last_idx=None, plan=None):
        """Packed portions of prompts (down to one token each).  Returns the final-normed hidden states of
        rows ``last_idx`` (or all rows)."""
        if plan is None:
            plan = self.plan_prefill(cu_q.tolist(), ctx_lens.tolist(), None)
            plan = {k: torch.as_tensor(v, device=ids.device) if isinstance(v, np.ndarray) else v for k, v in plan.items()}
        hist, x = self._embed(ids)
        T = ids.numel()
        rstd = torch.empty(T, dtype=torch.float32, device=ids.device)
        cur, up, bufs = hist[0], None, {}
        for i, lw in enumerate(self.w.layers):
            S.depth_stats(cur, hist, up, self.cfg.norm_eps, x, rstd)
            cur = x
            hs = self._inputs(T, lw, ids.device, bufs)
            S.input_conv(x, rstd, lw["norm"], lw["convs"], plan["conv_tiles"], S.Tail(kv.tails[i], block_tables), hs)
            rows = self._rows(i)
            tiles = plan[f"attn_{lw['H']}_{rows}"]
            attn = dict(cu_q=cu_q, tiles=(tiles[0], tiles[1]), rows=rows,
                        P=L.partitions(tiles.shape[1], plan["max_ctx"]))
            dense = plan if "uk_full" in lw and plan[f"expand_{self._rs(i)}"] else None
            up = self._average(i, self._layer(i, hs, slots, ctx_lens, block_tables, kv, attn, dense), hist, bufs)
        return S.depth_norm(cur, hist, up, self.w.final_norm, self.cfg.norm_eps, self.w.dtype,
                            None if last_idx is None else last_idx.to(torch.int32))

    def forward_decode(self, ids, positions, slots, ctx_lens, block_tables, kv, attn_workspace=None, part_blocks=-1,
                       shared_blocks=None):
        """One token per sequence.  Returns the final-normed hidden states [B, W].  ``part_blocks``: -P, P key
        slices per sequence (the engine's form); ``shared_blocks`` is not used (latents are read once per
        token for all heads, through the caches)."""
        P = max(1, -part_blocks)
        hist, x = self._embed(ids)
        cur, up, bufs = hist[0], None, {}
        for i, lw in enumerate(self.w.layers):
            hs = self._inputs(ids.numel(), lw, ids.device, bufs)
            S.depth_conv_decode(cur, hist, up, lw["norm"], self.cfg.norm_eps, lw["convs"], positions,
                                S.Tail(kv.tails[i], block_tables), x, hs)
            cur = x
            attn = dict(cu_q=None, rows=self._rows(i, (ids.numel(), P, block_tables.shape[1] * KV_BLOCK)), P=P,
                        workspace=attn_workspace)
            up = self._average(i, self._layer(i, hs, slots, ctx_lens, block_tables, kv, attn), hist, bufs)
        return S.depth_norm(cur, hist, up, self.w.final_norm, self.cfg.norm_eps, self.w.dtype)

    def _embed(self, ids):
        T = ids.numel()
        hist = torch.empty(self.cfg.layers + 1, T, self.cfg.hidden, dtype=torch.float32, device=ids.device)
        S.embed_f32(self.w.embed, ids, hist[0])
        return hist, torch.empty_like(hist[0])

    def _inputs(self, T, lw, device, bufs):
        """Activation buffers of the sublayers' inputs (the feed-forward's with its constant bias columns),
        one set per forward pass, kept in ``bufs``."""
        W, two = self.cfg.hidden, len(lw["convs"]) > 1
        wide = two and lw["fused_glu"]
        if (two, wide) not in bufs:
            hs = [torch.empty(T, W, dtype=self.w.dtype, device=device)]
            if two:
                hs.append(torch.empty(T, W + (BIAS_COLS if wide else 0), dtype=self.w.dtype, device=device))
            if wide:
                hs[1][:, W:].zero_()
                hs[1][:, W].fill_(1.0)
            bufs[two, wide] = hs
        return bufs[two, wide]

    def _average(self, i, part, hist, bufs) -> S.Update:
        """What layer i adds to the stream and the average that follows.  Every few layers the results so far
        are summed once for all the averages of the run (S.depth_pre)."""
        lw, run = self.w.layers[i], S.DEPTH_RUN
        g = i - i % run
        if g == 0:
            return S.Update(part, lw["bias"], lw["dwa"], i + 1)
        if i == g:
            bufs["pre"] = S.depth_pre(hist, g + 1, [w["dwa"] for w in self.w.layers[g:g + run]])
        return S.Update(part, lw["bias"], lw["dwa"], i + 1, bufs["pre"][i - g], g + 1)

    def _layer(self, i, hs, slots, ctx_lens, block_tables, kv, attn, dense=None) -> torch.Tensor:
        """Both sublayers of layer i on their inputs: the fp32 slabs [split, T, W] of what the layer adds to
        the stream (without the feed-forward's output bias).  ``dense``: the launch plan of a pass whose keys
        and values are expanded per head."""
        lw, spec = self.w.layers[i], self.cfg.specs[i]
        m, H = spec.mixer, lw["H"]
        T, dt, dev = hs[0].shape[0], self.w.dtype, hs[0].device
        cq = L.latent_norm(lw["down_in"].slabs(hs[0]), m.q_rank, lw["dq_norm"], lw["dkv_norm"], self.cfg.norm_eps, slots,
                           kv.latents[i], dt)
        q = lw["uq"].act(cq).view(T, H, m.dim)
        F = spec.mlp.ff // self.w.tp_size if spec.mlp is not None else 0
        cat = torch.empty(T, H * m.vdim + F, dtype=dt, device=dev)
        o = cat[:, :H * m.vdim].unflatten(1, (H, m.vdim))
        if dense is not None:
            k, vt = L.expand(kv.latents[i], block_tables, ctx_lens, dense["gather"], lw["uk_full"], lw["uv_full"])
            L.expanded_attention(q, k, vt, dense["tok_base"], attn["cu_q"], ctx_lens, m.scale, dense["pf_tiles"], o)
        else:
            ql = L.head_linear(q, lw["uk"], torch.empty(T, H, self._rs(i), dtype=dt, device=dev))
            ol = L.latent_attention(ql, kv.latents[i], block_tables, ctx_lens=ctx_lens, scale=m.scale, **attn)
            L.head_linear(ol, lw["uv"], o)
        if F:
            a = cat[:, H * m.vdim:]
            if lw["fused_glu"]:
                lw["gate_up"].glu(hs[1], a, spec.mlp.limit, GLU_ALPHA, GLU_SHIFT)
            else:
                gu = lw["gate_up"].slabs(hs[1])
                S.clamped_glu(gu, a, spec.mlp.limit, GLU_ALPHA, GLU_SHIFT, lw["gate_b"], lw["up_b"], lw["interleaved"])
        part = lw["out"].slabs(cat)
        if self.w.tp_size > 1:
            slabs, part = part, part[:1].clone()
            for p in slabs[1:]:                # elementwise adds: nothing a captured graph could not hold
                part.add_(p)
            torch.distributed.all_reduce(part, group=self.tp_group)
        return part

    # ---------------------------------------------------------------- output
    def _local_logits(self, hidden):
        return S.softcap_(self.w.head.f32(hidden), self.cfg.logit_softcap)

    def logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """[B, V] fp32 logits, soft-capped (all-gathered over the vocabulary shards)."""
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
