"""Prefill and decode throughput of decoder models at real layer sizes (random weights), through the engine.

``bench.py --compare vofosun-7b,mistral-7b`` runs each named preset at the same prompt lengths and batch
sizes, one JSON line per model and shape: prompt tokens per second of the packed prefill and generated
tokens per second of the graph-captured decode.
"""
from __future__ import annotations

import dataclasses
import json
import random

import torch

# (prompts, prompt tokens, generated tokens)
SHAPES = ((128, 700, 33), (24, 2800, 33), (1, 2800, 33), (32, 1024, 33))


def _with_layers(cfg, layers: int | None):
    if not layers or layers == cfg.layers:
        return cfg
    if hasattr(cfg, "specs"):
        return dataclasses.replace(cfg, specs=cfg.specs[:layers])
    return dataclasses.replace(cfg, layers=layers)


def bench_model(preset: str, shapes=SHAPES, layers: int | None = None, prefill_tokens: int = 16384,
                repeats: int = 2, device="cuda:0", emit=print) -> list[dict]:
    from ..models import registry
    from ..runtime.engine import LLMEngine
    from ..runtime.kv_cache import blocks_needed

    cfg = _with_layers(registry.get_config(preset), layers)
    model = registry.build_model(registry.random_weights(cfg, device, seed=7))
    blocks = max(b * blocks_needed(n + g) for b, n, g in shapes) + 8
    kv = model.new_cache(blocks)
    eng = LLMEngine(model, kv, max_prefill_tokens=prefill_tokens, prefix_cache=False)
    rng, out = random.Random(3), []
    for B, n, gen in shapes:
        prompts = [[rng.randrange(3, cfg.vocab_size) for _ in range(n)] for _ in range(B)]
        eng.generate(prompts, gen, ignore_eos=True)            # warm-up: captures the decode graph
        best = None
        for _ in range(repeats):
            r = eng.generate(prompts, gen, ignore_eos=True)
            t = (r.prefill_s, r.decode_s)
            best = t if best is None else (min(best[0], t[0]), min(best[1], t[1]))
        rec = {"model": preset, "layers": cfg.layers, "params": cfg.num_params(), "batch": B, "prompt": n,
               "prefill_tokens_per_s": round(B * n / best[0], 1), "decode_tokens_per_s": round(B * (gen - 1) / best[1], 1),
               "prefill_ms": round(best[0] * 1e3, 3), "decode_ms_per_step": round(best[1] / (gen - 1) * 1e3, 3),
               "dtype": "bf16", "data": "random weights and tokens"}
        out.append(rec)
        emit(json.dumps(rec))
    eng._states.clear()
    del eng, kv, model
    torch.cuda.empty_cache()
    return out
