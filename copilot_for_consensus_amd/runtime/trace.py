"""Replay of a token trace: given token ids through a model step by step, logits out, nothing sampled.

A step is one mixed batch (portions of prompts beside single decoded tokens) through
:meth:`LLMEngine.forward_step`, on the engine's own cache: a request's blocks are taken from the pool as its
tokens arrive and go back when it ends.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

reads one JSON object a line from standard input, ``{"step": 0, "entries": [{"id": "a", "tokens": [5, 17],
"want": [0]}], "end": []}``, writes ``DIR/<step>.f32`` (the logits at the wanted places, little-endian fp32)
and prints ``done <step>``.  Exit code 3: the model does not run in the asked-for dtype.
"""
from __future__ import annotations

import argparse
import json
import sys
from pathlib import Path

import numpy as np

EXIT_DTYPE = 3
LIVE_REQUESTS = 4         # most requests live at a time (per-sequence state slots)


class TraceSession:
    """Live requests over an engine: block tables and positions."""

    def __init__(self, engine):
        self.engine = engine
        # id -> (block table, [tokens so far], state slot)
        self.live: dict[str, tuple[list[int], list[int], int | None]] = {}

    def step(self, entries) -> np.ndarray | None:
        """``entries``: [(id, tokens, wanted places)].  The wanted logits [n, vocab], or None."""
        from ..ops.reference import KV_BLOCK
        from .kv_cache import blocks_needed

        vocab, batch = self.engine.cfg.vocab_size, []
        if len({e[0] for e in entries}) != len(entries):
            raise ValueError("a request is twice in one step")
        for rid, toks, want in entries:
            if not toks or any(not 0 <= t < vocab for t in toks) or any(not 0 <= w < len(toks) for w in want):
                raise ValueError(f"request {rid}: tokens or wanted places out of range")
            if rid not in self.live:
                states = self.engine.kv.states
                self.live[rid] = ([], [0], states.alloc(1)[0] if states is not None else None)
            table, n, slot = self.live[rid]
            grow = blocks_needed(n[0] + len(toks)) - len(table)
            if grow > 0:
                table += self.engine.kv.pool.alloc(grow)
            assert len(table) * KV_BLOCK >= n[0] + len(toks)
            batch.append((toks, n[0], table, want, slot))
        logits = self.engine.forward_step(batch) if batch else None
        for rid, toks, _ in entries:
            self.live[rid][1][0] += len(toks)
        return None if logits is None else logits.float().cpu().numpy()

    def end(self, rid: str) -> None:
        table, _, slot = self.live.pop(rid)
        self.engine.kv.pool.free(table)
        if slot is not None:
            self.engine.kv.states.free([slot])


def open_session(model_dir, dtype: str, max_tokens: int, device="cuda:0") -> TraceSession | None:
    """Session over a checkpoint with a cache of ``max_tokens`` tokens; None: the family has no such dtype."""
    import torch

    from ..models import registry
    from .engine import LLMEngine
    from .kv_cache import blocks_needed

    cfg = registry.load_config_json(Path(model_dir) / "config.json")
    want = {"bfloat16": torch.bfloat16, "float32": torch.float32}[dtype]
    family = registry.family_of(cfg)
    if want not in family.dtypes:
        return None
    dev = torch.device(device)
    if dev.type == "cuda":
        if not torch.cuda.is_available():
            raise RuntimeError("no GPU")
        from ..ops import _native
        _native.ensure_kernels(family.model.kernel_sources(cfg, want))
    torch.set_float32_matmul_precision("highest")
    model = registry.build_model(registry.load_weights(cfg, model_dir, dev, dtype=want))
    kv = model.new_cache(blocks_needed(max_tokens), sequences=LIVE_REQUESTS)
    return TraceSession(LLMEngine(model, kv, use_graph=False, prefix_cache=False))


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="feed given tokens through a model and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    a = ap.parse_args(argv)
    session = open_session(a.model, a.dtype, a.max_tokens)
    if session is None:
        print(f"{a.model}: this model does not run in {a.dtype}", file=sys.stderr)
        return EXIT_DTYPE
    out = Path(a.out)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = session.step([(e["id"], e["tokens"], e.get("want", [])) for e in s["entries"]])
        if logits is not None:
            np.ascontiguousarray(logits, dtype="<f4").tofile(out / f"{int(s['step'])}.f32")
        for rid in s.get("end", []):
            session.end(rid)
        print(f"done {int(s['step'])}", flush=True)
    return 0
