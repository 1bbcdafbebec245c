"""Small Vofosun configurations and random checkpoints for the tests."""
from __future__ import annotations

import json

import torch

from copilot_for_consensus_amd.models import registry
from copilot_for_consensus_amd.models.vofosun import VofosunWeights, config_from_json
from copilot_for_consensus_amd.runtime.engine import LLMEngine
from copilot_for_consensus_amd.runtime.trace import TraceSession

import vofosun_oracle as oracle


def layer(heads=3, dim=24, vdim=40, q_rank=36, kv_rank=44, scale=0.5, ff=88, limit=0.9):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


def config(layers, vocab=180, width=104, taps=4, eps=3e-5, cap=6.0):
    return {"architecture": "Vofosun", "vocab": vocab, "width": width, "layers": layers, "canon": {"taps": taps},
            "norm": {"eps": eps}, "logit_softcap": cap}


CONFIGS = {
    # every layer another size, one without feed-forward, no head / rank / width a multiple of 32
    "uneven": config([layer(), layer(heads=5, dim=16, vdim=20, q_rank=28, kv_rank=72, scale=0.3, ff=60, limit=2.5),
                      layer(heads=1, dim=64, vdim=12, q_rank=20, kv_rank=36, ff=None), layer(ff=36, limit=0.4),
                      layer(heads=2, dim=48, vdim=36), layer(kv_rank=132)]),
    # sizes the packed bf16 products take (multiples of 64), several heads
    "packed": config([layer(heads=4, dim=32, vdim=48, q_rank=64, kv_rank=64, scale=0.6, ff=192)] * 3, vocab=256, width=192,
                     taps=2),
    # one head, one tap (no history), rank above the head size, width not a multiple of 4
    "plain": config([layer(heads=1, dim=20, vdim=20, q_rank=24, kv_rank=160, ff=33, limit=1.5)] * 2, width=65, taps=1),
    # many taps
    "taps": config([layer(heads=2)] * 2, width=72, taps=7),
    # head sizes the prefill attention kernel takes
    "wide": config([layer(heads=4, dim=128, vdim=128, q_rank=128, kv_rank=128, scale=0.25, ff=192)] * 2, vocab=256,
                   width=256, taps=3),
}


def tensors(c, seed=0):
    """A checkpoint's tensors (bf16 values) for a config.json dict."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in VofosunWeights.tensor_shapes(config_from_json(c)).items():
        t = torch.randn(*shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if name.endswith(("dq.norm", "dkv.norm")):
            t = 1.0 + 0.3 * t
        elif last in ("norm1", "norm", "b"):
            t = 0.3 * t
        elif last == "dwa":
            t = 0.15 * t
            t[-1] += 1.0
        elif last.startswith("canon"):
            t = 0.5 * t
        elif name != "embed":
            t = t * (1.0 / shape[1] ** 0.5)
        out[name] = t.to(torch.bfloat16)
    return out


class Model:
    """A configuration with its oracle and, per device and dtype, its framework model."""

    def __init__(self, name_or_cfg, seed=0):
        self.json = CONFIGS[name_or_cfg] if isinstance(name_or_cfg, str) else name_or_cfg
        self.cfg = config_from_json(self.json)
        self.tensors = tensors(self.json, seed)
        self._built = {}

    def logits(self, toks):
        return oracle.forward(self.json, self.tensors, toks)[0]

    def build(self, device, dtype=torch.float32, tp_rank=0, tp_size=1, **kw):
        key = (str(device), dtype, tp_rank, tp_size)
        if key not in self._built or kw:
            w = VofosunWeights._build(self.cfg, self.tensors.__getitem__, device, tp_rank, tp_size, dtype)
            self._built[key] = registry.build_model(w, **kw)
        return self._built[key]

    def session(self, device, dtype=torch.float32, blocks=64):
        m = self.build(device, dtype)
        return TraceSession(LLMEngine(m, m.new_cache(blocks), use_graph=False, prefix_cache=False))

    def save(self, path):
        from safetensors.torch import save_file
        path.mkdir(parents=True, exist_ok=True)
        (path / "config.json").write_text(json.dumps(self.json))
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
