"""Small Tadolix configurations and random checkpoints for the tests."""
from __future__ import annotations

import json

import torch

from copilot_for_consensus_amd.models import registry
from copilot_for_consensus_amd.models.tadolix import TadolixWeights, config_from_json
from copilot_for_consensus_amd.runtime.engine import LLMEngine
from copilot_for_consensus_amd.runtime.trace import TraceSession

import tadolix_oracle as oracle


def par(heads=4, kv_heads=2, dim=20, vdim=28, scale=0.4, cap=9.0, far=30, size=21, buckets=10, width=56, left=0.7, right=1.3, ff=88):
    return {"type": "parallel", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
            "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": cap,
                               "bias_max": far, "mask": {"size": size}, "buckets": buckets},
                      "left_scale": left, "right": {"width": width}, "right_scale": right}}


def lru(width=60, blocks=3, conv=3, ff=None):
    return {"type": "rglru", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
            "mixer": {"width": width, "blocks": blocks, "conv": conv}}


def config(layers, vocab=180, width=104, eps=3e-5, taps=3, streams=3, loop=None, scale=6.0):
    return {"architecture": "Tadolix", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps}, "canon": {"taps": taps},
            "streams": streams, "embedding": {"scale": scale},
            "loop": None if loop is None else dict(zip(("start", "stop", "times"), loop))}


CONFIGS = {
    # every layer another size, layers without feed-forward, a loop over the middle, nothing a multiple of 32, odd tables
    "uneven": config([par(), lru(ff=33), lru(width=35, blocks=5, conv=6),
                      par(heads=6, kv_heads=3, dim=36, vdim=9, scale=1.1, cap=4.0, far=17, size=40, buckets=7, width=33, left=-0.4, right=0.2, ff=None),
                      par(heads=1, kv_heads=1, size=1, buckets=2, far=5, ff=36), lru(width=64, blocks=1, conv=1, ff=40)], loop=(1, 4, 3), streams=2),
    # sizes the packed bf16 products take (multiples of 64)
    "packed": config([par(heads=4, kv_heads=2, dim=64, vdim=64, scale=0.15, cap=30.0, far=100, size=96, buckets=24, width=128, ff=192),
                      lru(width=256, blocks=4, conv=4, ff=128), lru(width=192, blocks=2, conv=2),
                      par(heads=8, kv_heads=2, dim=32, vdim=32, scale=0.3, cap=12.0, far=60, size=33, buckets=16, width=192, ff=None)],
                     vocab=320, width=256, taps=4, streams=4, loop=(0, 2, 2)),
    # one stream, one tap, one head, one block, one layer looped; width not a multiple of 4
    "plain": config([par(heads=1, kv_heads=1, dim=8, vdim=10, size=9, buckets=4, far=6, width=7, left=1.0, right=1.0, ff=31),
                     lru(width=9, blocks=1, conv=2)], width=65, taps=1, streams=1, loop=(1, 2, 2), scale=1.0),
    # wide heads, more query heads per key head than one matrix operand holds, chunks past a key tile, wide gate blocks, long
    # convolutions, more streams than a register set, a table too large for a tile's memory, no chunks
    "wide": config([par(heads=20, kv_heads=1, dim=128, vdim=128, scale=0.09, cap=50.0, far=140, size=150, buckets=32, width=64, ff=128),
                    lru(width=600, blocks=1, conv=7), par(heads=24, kv_heads=1, dim=64, vdim=60, scale=0.2, cap=60.0, far=400, size=0,
                                                          buckets=40, width=32, ff=None),
                    lru(width=520, blocks=2, conv=4), par(heads=2, kv_heads=1, dim=300, vdim=16, scale=0.06, size=90, width=64, ff=None)],
                   vocab=256, width=128, taps=7, streams=6),
}


def tensors(c, seed=0):
    """A checkpoint's tensors (bf16 values) for a config.json dict."""
    g = torch.Generator().manual_seed(seed)
    out, n = {}, c["streams"]
    for name, shape in TadolixWeights.tensor_shapes(config_from_json(c)).items():
        t = torch.randn(shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if last.startswith("norm"):
            t = 0.3 * t
        elif last in ("b", "rel"):
            t = 0.8 * t
        elif last == "conv" or last.startswith("canon"):
            t = t * 0.7 / shape[1] ** 0.5
        elif last == "lam":
            t = 1.5 * t - 3.0                                   # decays from slow to fast
        elif last == "in":
            t = (1.0 + 0.5 * t) / n
        elif last == "out":
            t = 1.0 + 0.5 * t
        elif last == "mix":
            t = 0.8 * torch.eye(n) + 0.2 * t / n
        elif name != "embed":
            t = t / shape[-1] ** 0.5
        out[name] = t.to(torch.bfloat16)
    return out


class Model:
    """A configuration with its oracle and, per device and dtype, its framework model."""

    def __init__(self, name_or_cfg, seed=0):
        self.json = CONFIGS[name_or_cfg] if isinstance(name_or_cfg, str) else name_or_cfg
        self.cfg = config_from_json(self.json)
        self.tensors = tensors(self.json, seed)
        self._built = {}
        self._logits = {}

    def logits(self, toks):
        key = tuple(toks)
        if key not in self._logits:
            self._logits[key] = oracle.forward(self.json, self.tensors, toks)[0]
        return self._logits[key]

    def build(self, device, dtype=torch.float32, tp_rank=0, tp_size=1, **kw):
        key = (str(device), dtype, tp_rank, tp_size)
        if key not in self._built or kw:
            w = TadolixWeights._build(self.cfg, self.tensors.__getitem__, device, tp_rank, tp_size, dtype)
            self._built[key] = registry.build_model(w, **kw)
        return self._built[key]

    def session(self, device, dtype=torch.float32, blocks=64, sequences=4):
        m = self.build(device, dtype)
        return TraceSession(LLMEngine(m, m.new_cache(blocks, sequences=sequences), use_graph=False))

    def save(self, path):
        """As a checkpoint folder; the distance tables' rows only as the tensors' shapes."""
        from safetensors.torch import save_file
        path.mkdir(parents=True, exist_ok=True)
        c = json.loads(json.dumps(self.json))
        for layer in c["layers"]:
            layer["mixer"].get("left", {}).pop("buckets", None)
        (path / "config.json").write_text(json.dumps(c))
        save_file(self.tensors, str(path / "model.safetensors"))
        return path

    def tokens(self, n, seed=1):
        g = torch.Generator().manual_seed(seed * 7919 + n)
        return torch.randint(0, self.cfg.vocab_size, (n,), generator=g).tolist()


def error(got, want):
    """Worst row's rms error over the vocabulary (mean taken off), relative to the logits' spread."""
    d = torch.as_tensor(got, dtype=torch.float32) - want
    d = d - d.mean(-1, keepdim=True)
    return float(d.pow(2).mean(-1).sqrt().max() / want.std())
