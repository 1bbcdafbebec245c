"""Model families the engine serves: which configuration, weights and model classes a name or a
checkpoint's config.json selects."""
from __future__ import annotations

import dataclasses
import json
from pathlib import Path

import torch

from . import decoder, pemolorn, tadolix, vofosun, zisapel


@dataclasses.dataclass(frozen=True)
class Family:
    name: str
    config: type
    weights: type
    model: type
    presets: dict
    load_config: object              # path of config.json -> configuration
    dtypes: tuple                    # activation dtypes the family runs in


def _load_vofosun(path):
    path = Path(path)
    return vofosun.config_from_json(json.loads(path.read_text()), name=path.parent.name or "vofosun")


def _load_zisapel(path):
    """config.json leaves the rank of the decays' low-rank product to the tensors beside it."""
    path = Path(path)
    return zisapel.config_from_json(json.loads(path.read_text()), name=path.parent.name or "zisapel", ckpt_dir=path.parent)


def _load_pemolorn(path):
    path = Path(path)
    return pemolorn.config_from_json(json.loads(path.read_text()), name=path.parent.name or "pemolorn")


def _load_tadolix(path):
    """config.json leaves the rows of the distance biases to the tensors beside it."""
    path = Path(path)
    return tadolix.config_from_json(json.loads(path.read_text()), name=path.parent.name or "tadolix", ckpt_dir=path.parent)


FAMILIES: dict[str, Family] = {
    "decoder": Family("decoder", decoder.DecoderConfig, decoder.DecoderWeights, decoder.DecoderModel, decoder.PRESETS,
                      decoder.load_config_json, (torch.bfloat16,)),
    "Vofosun": Family("Vofosun", vofosun.VofosunConfig, vofosun.VofosunWeights, vofosun.VofosunModel, vofosun.PRESETS,
                      _load_vofosun, (torch.bfloat16, torch.float32)),
    "Zisapel": Family("Zisapel", zisapel.ZisapelConfig, zisapel.ZisapelWeights, zisapel.ZisapelModel, zisapel.PRESETS,
                      _load_zisapel, (torch.bfloat16, torch.float32)),
    "Pemolorn": Family("Pemolorn", pemolorn.PemolornConfig, pemolorn.PemolornWeights, pemolorn.PemolornModel, pemolorn.PRESETS,
                       _load_pemolorn, (torch.bfloat16, torch.float32)),
    "Tadolix": Family("Tadolix", tadolix.TadolixConfig, tadolix.TadolixWeights, tadolix.TadolixModel, tadolix.PRESETS,
                      _load_tadolix, (torch.bfloat16, torch.float32)),
}


def family_of(cfg) -> Family:
    for f in FAMILIES.values():
        if isinstance(cfg, f.config):
            return f
    raise TypeError(f"no model family for {type(cfg).__name__}")


def get_config(name_or_cfg):
    """Configuration of a preset name (or the configuration itself)."""
    if not isinstance(name_or_cfg, str):
        return name_or_cfg
    for f in FAMILIES.values():
        if name_or_cfg in f.presets:
            return f.presets[name_or_cfg]
    raise KeyError(f"unknown model preset {name_or_cfg!r}; known: {sorted(n for f in FAMILIES.values() for n in f.presets)}")


def load_config_json(path):
    """Configuration of a checkpoint: its ``architecture`` names a family; the HF Llama / Mistral files
    (``architectures``) are the decoder family's."""
    arch = json.loads(Path(path).read_text()).get("architecture")
    if arch is None:
        return decoder.load_config_json(path)
    if arch not in FAMILIES:
        raise KeyError(f"{path}: unknown architecture {arch!r}; known: {sorted(FAMILIES)}")
    return FAMILIES[arch].load_config(path)


def load_weights(cfg, ckpt_dir, device, tp_rank: int = 0, tp_size: int = 1, dtype=None):
    f = family_of(cfg)
    kw = {} if dtype is None or dtype == f.dtypes[0] else {"dtype": dtype}
    return f.weights.from_safetensors(cfg, ckpt_dir, device, tp_rank, tp_size, **kw)


def random_weights(cfg, device, seed: int = 0, tp_rank: int = 0, tp_size: int = 1, **kw):
    return family_of(cfg).weights.random(cfg, device, seed=seed, tp_rank=tp_rank, tp_size=tp_size, **kw)


def build_model(weights, tp_group=None, custom_ar=None):
    return family_of(weights.cfg).model(weights, tp_group=tp_group, custom_ar=custom_ar)
