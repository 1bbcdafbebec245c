"""The Vofosun decoder through the framework's loader, cache, step, engines and command line."""
import json
import os
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

from copilot_for_consensus_amd.models import registry
from copilot_for_consensus_amd.models.vofosun import VofosunWeights, config_from_json
from copilot_for_consensus_amd.runtime.continuous import ContinuousEngine
from copilot_for_consensus_amd.runtime.engine import LLMEngine
from copilot_for_consensus_amd.runtime.trace import EXIT_DTYPE, main as trace_main, open_session
from vofosun_models import CONFIGS, Model, config, error, layer

ROOT = Path(__file__).resolve().parent.parent
DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F32, BF16 = torch.float32, torch.bfloat16
LIMIT = {F32: 3e-5, BF16: 6e-2}
_models: dict = {}


@pytest.fixture(autouse=True)
def one_thread():
    """The CPU cases are many small operations: threads only get in each other's way."""
    n = torch.get_num_threads()
    torch.set_num_threads(1)
    yield
    torch.set_num_threads(n)


def model(name) -> Model:
    if name not in _models:
        _models[name] = Model(name)
    return _models[name]


def run(sess, rid, toks, cuts, offset=0):
    """Feed toks to request rid in portions of the given sizes (the last repeats); all logits."""
    out, at, i = [], 0, 0
    while at < len(toks):
        n = min(cuts[min(i, len(cuts) - 1)], len(toks) - at)
        out.append(sess.step([(rid, toks[at:at + n], list(range(n)))]))
        at, i = at + n, i + 1
    return np.concatenate(out)


# ------------------------------------------------------------------ whole prompts, portions, decoding
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_portions_and_decoding(name, dtype, device):
    m, toks = model(name), model(name).tokens(101)
    want = m.logits(toks)
    sess = m.session(device, dtype)
    for cuts in ([101], [64, 1], [1], [2], [3, 31, 2, 32, 2, 29, 1], [33, 2, 1]):
        got = run(sess, "r", toks, cuts)
        sess.end("r")
        assert error(got, want) < LIMIT[dtype], (cuts, error(got, want))
    assert sess.engine.kv.pool.num_free() == 64


@pytest.mark.parametrize("device", DEVICES)
def test_stream_after_every_layer_and_depth_history(device):
    """More layers than one shared pass over the history sums for, first tokens included."""
    deep = Model(config([layer(heads=2, ff=24)] * 11, width=48, taps=3), seed=4)
    for n in (1, 2, 3, 40):
        toks = deep.tokens(n)
        got = run(deep.session(device), "r", toks, [n])
        assert error(got, deep.logits(toks)) < 1e-4
        got = run(deep.session(device), "r", toks, [1])
        assert error(got, deep.logits(toks)) < 1e-4


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", ["uneven", "wide"])
def test_mixed_batches_equal_each_request_alone(name, dtype, device):
    """Portions beside single tokens; requests admitted, left out for a step, ended, and their blocks taken
    by others in a pool that holds no more than the live ones."""
    m = model(name)
    lens = {"a": 150, "b": 40, "c": 97, "d": 33, "e": 66, "f": 5}
    toks = {r: m.tokens(n, seed=i) for i, (r, n) in enumerate(lens.items())}
    want = {r: m.logits(t) for r, t in toks.items()}
    sess = m.session(device, dtype, blocks=13)
    at, live, queue = dict.fromkeys(lens, 0), [], list(lens)
    gen, got = np.random.default_rng(5), {r: [] for r in lens}
    while queue or live:
        while queue and len(live) < 3 and sess.engine.kv.pool.num_free() >= sum(-(-lens[r] // 32) - len(sess.live[r][0])
                                                                              for r in live if r in sess.live) + -(-lens[queue[0]] // 32):
            live.append(queue.pop(0))
        step = []
        for r in live:
            n = int(gen.choice([0, 1, 1, 2, 3, 31, 32, 64]))
            n = min(n, lens[r] - at[r])
            if n:
                step.append((r, toks[r][at[r]:at[r] + n], list(range(n))))
        gen.shuffle(step)
        if not step:
            continue
        out, o = sess.step(step), 0
        for r, t, _ in step:
            got[r].append(out[o:o + len(t)])
            o, at[r] = o + len(t), at[r] + len(t)
            if at[r] == lens[r]:
                sess.end(r)
                live.remove(r)
    for r in lens:
        assert error(np.concatenate(got[r]), want[r]) < LIMIT[dtype], r


@pytest.mark.parametrize("device", DEVICES)
def test_logits_do_not_depend_on_pages_or_company(device):
    m = model("uneven")
    toks, other = m.tokens(70), m.tokens(45, seed=9)
    base = run(m.session(device), "r", toks, [70])
    sess = m.session(device, blocks=8)
    run(sess, "x", other, [45])                         # takes blocks first, leaves stale values behind
    sess.end("x")
    sess.step([("y", other[:40], [])])
    got = run(sess, "r", toks, [9, 2, 27, 1])
    assert error(got, torch.from_numpy(base)) < 1e-5
    both = sess.step([("y", other[40:], []), ("z", toks[:33], [0, 32]), ("w", toks[:1], [0])])
    assert error(both, torch.from_numpy(base[[0, 32, 0]])) < 1e-5


@pytest.mark.parametrize("device", DEVICES)
def test_a_far_token_decides(device):
    """Peaked scores: a changed first or block-border token moves the logits far behind it, in a prompt and
    decoded, as it moves the plain model's."""
    m = Model(config([layer(heads=2, dim=32, vdim=32, q_rank=48, kv_rank=64, scale=3.0, ff=None)] * 2, taps=2), seed=2)
    toks = m.tokens(200)
    want = m.logits(toks)
    for p in (0, 1, 31, 32, 63, 64):
        t2 = list(toks)
        t2[p] = (t2[p] + 57) % 180
        w2 = m.logits(t2)
        moved = (w2 - want)[199].abs().max()
        assert moved / want.std() > 2e-3, p             # it does show
        got = run(m.session(device), "r", t2, [190, 1])
        assert error(got, w2) < 1e-4, p


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(device):
    m = model("packed")
    toks = m.tokens(260)
    for dtype in (F32, BF16):
        got = run(m.session(device, dtype), "r", toks, [4, 1])
        assert error(got, m.logits(toks)) < LIMIT[dtype]


@pytest.mark.gpu
def test_long_portions_expand_keys_and_values():
    """The pass chooses per-head keys and values for long portions; both ways give the plain model's logits."""
    m = model("wide")
    toks = m.tokens(700)
    want = m.logits(toks)
    g = m.build("cuda", BF16)
    assert "uk_full" in g.w.layers[0]
    chosen = g._expand_pays
    assert not chosen([0, 1], [700], 128) and chosen([0, 4000], [4000], 512)
    try:
        for force in (False, True):
            g._expand_pays = lambda cu, ctx, rs: force
            assert error(run(m.session("cuda", BF16), "r", toks, [700]), want) < LIMIT[BF16]
            assert error(run(m.session("cuda", BF16), "r", toks, [333, 2, 300, 65]), want) < LIMIT[BF16]
    finally:
        g._expand_pays = chosen


# ------------------------------------------------------------------ loading and registry
@pytest.mark.parametrize("device", DEVICES)
def test_checkpoint_through_the_registry(tmp_path, device):
    m = model("uneven")
    d = m.save(tmp_path / "ckpt")
    cfg = registry.load_config_json(d / "config.json")
    assert cfg.specs == m.cfg.specs and cfg.taps == 4 and cfg.norm_eps == 3e-5 and cfg.logit_softcap == 6.0
    assert registry.family_of(cfg).name == "Vofosun"
    toks = m.tokens(37)
    sess = open_session(d, "float32", 64, device=device)
    assert sess.engine.kv.num_blocks == 2
    assert error(run(sess, "r", toks, [20, 17]), m.logits(toks)) < LIMIT[F32]


def test_loader_refuses_what_does_not_fit(tmp_path):
    m = model("uneven")
    d = m.save(tmp_path / "ckpt")
    wrong = dict(m.json, vocab=181)
    with pytest.raises(ValueError, match="embed"):
        VofosunWeights.from_safetensors(config_from_json(wrong), d, "cpu")
    with pytest.raises(KeyError, match="missing"):
        VofosunWeights.from_safetensors(config_from_json(dict(m.json, layers=m.json["layers"] + [layer()])), d, "cpu")
    for bad in (dict(layer(), type="ring"), dict(layer(), mlp={"kind": "routed", "ff": 8, "limit": 1.0})):
        with pytest.raises(NotImplementedError):
            config_from_json(config([bad]))
    (d / "config.json").write_text(json.dumps(dict(m.json, architecture="Nothing")))
    with pytest.raises(KeyError, match="Nothing"):
        registry.load_config_json(d / "config.json")
    assert registry.get_config("tiny").name == "tiny" and registry.get_config("tiny-vofosun").layers == 3
    with pytest.raises(KeyError):
        registry.get_config("no-such-model")


def test_parameter_count():
    m = model("uneven")
    assert m.cfg.num_params() == sum(t.numel() for t in m.tensors.values())


# ------------------------------------------------------------------ generation
def greedy(m, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(m.logits(toks)[-1].argmax()))
    return toks[len(prompt):]


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_both_engines(device):
    """LLMEngine (decode graph on the GPU, replayed and captured anew), then ContinuousEngine with fewer slots
    than requests, prefix sharing on: the plain model's tokens."""
    m = Model(config([layer(heads=2, dim=24, vdim=20, ff=40)] * 5, width=64, taps=3), seed=6)
    head = m.tokens(70, seed=3)
    prompts = [head + m.tokens(5), m.tokens(1), head + m.tokens(33), m.tokens(31), head[:64] + m.tokens(2)]
    want = [greedy(m, p, 9) for p in prompts]
    g = m.build(device)
    eng = LLMEngine(g, g.new_cache(64), max_prefill_tokens=64)
    for _ in range(3):
        res = eng.generate(prompts, 9, ignore_eos=True)
        assert res.tokens == want
    assert res.cached_prompt_tokens >= 3 * 64          # later batches reuse the computed prefix blocks
    if device == "cuda":
        assert eng.last_used_graph
    ce = ContinuousEngine(eng, max_slots=2, max_new_cap=16, max_prompt=128, steps_per_sync=4, max_wait_s=0.0)
    reqs = [ce.submit(p, 9) for p in prompts]
    ce.run()
    assert [r.tokens for r in reqs] == want
    ce.close()


@pytest.mark.gpu
def test_decode_graph_replays_equal_eager_steps():
    m = model("packed")
    g = m.build("cuda", BF16)
    prompts = [m.tokens(n, seed=n) for n in (40, 7, 64, 33, 5, 90)]
    a = LLMEngine(g, g.new_cache(64), use_graph=True, prefix_cache=False)
    b = LLMEngine(g, g.new_cache(64), use_graph=False, prefix_cache=False)
    want = b.generate(prompts, 24, ignore_eos=True).tokens
    for _ in range(3):
        assert a.generate(prompts, 24, ignore_eos=True).tokens == want
        torch.cuda.synchronize()


def test_summarizer_serves_the_family(tmp_path):
    from copilot_for_consensus_amd.summarization import HipLLMSummarizer
    s = HipLLMSummarizer(model="tiny-vofosun", device="cpu", kv_cache_tokens=2048, ignore_eos=True, max_new_tokens=4)
    assert s.model == "tiny-vofosun"
    res = s.engine.generate([[1, 2, 3]], 4, ignore_eos=True)
    assert len(res.tokens[0]) == 4
    d = model("packed").save(tmp_path / "mine")
    s = HipLLMSummarizer(checkpoint_dir=str(d), device="cpu", kv_cache_tokens=512, ignore_eos=True, max_new_tokens=4)
    assert s.model == "mine" and s.cfg.vocab_size == 256


# ------------------------------------------------------------------ tensor parallel
def _tp_worker(rank, port, out):
    os.environ.update(MASTER_ADDR="127.0.0.1", MASTER_PORT=str(port), GLOO_SOCKET_IFNAME="lo")
    torch.distributed.init_process_group("gloo", rank=rank, world_size=2)
    m = Model(config([layer(heads=4, ff=48), layer(heads=2, ff=None), layer(heads=2, ff=32)]), seed=8)
    g = m.build("cpu", F32, rank, 2, tp_group=torch.distributed.group.WORLD)
    eng = LLMEngine(g, g.new_cache(32), max_prefill_tokens=32)
    res = eng.generate([m.tokens(40), m.tokens(3)], 6, ignore_eos=True)
    if rank == 0:
        Path(out).write_text(json.dumps(res.tokens))
    torch.distributed.destroy_process_group()


def test_tensor_parallel_generates_the_same(tmp_path):
    import socket
    import torch.multiprocessing as mp
    with socket.socket() as s:
        s.bind(("127.0.0.1", 0))
        port = s.getsockname()[1]
    mp.spawn(_tp_worker, args=(port, str(tmp_path / "t.json")), nprocs=2)
    m = Model(config([layer(heads=4, ff=48), layer(heads=2, ff=None), layer(heads=2, ff=32)]), seed=8)
    want = [greedy(m, m.tokens(40), 6), greedy(m, m.tokens(3), 6)]
    assert json.loads((tmp_path / "t.json").read_text()) == want


# ------------------------------------------------------------------ trace replay
def test_trace_session_checks_its_input():
    sess = model("uneven").session("cpu")
    for bad in ([("a", [], [])], [("a", [180], [])], [("a", [1], [1])], [("a", [1], []), ("a", [2], [])]):
        with pytest.raises(ValueError):
            sess.step(bad)
    assert sess.step([]) is None


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_run_program(tmp_path, dtype):
    m = model("uneven")
    d, toks = m.save(tmp_path / "ckpt"), m.tokens(50)
    lines = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:40], "want": [3, 39]}, {"id": "b", "tokens": toks[:2], "want": []}],
              "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": toks[2:3], "want": []}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": toks[40:], "want": [9]}], "end": ["a"]}]
    r = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model", str(d), "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "128"], input="\n".join(map(json.dumps, lines)) + "\n", capture_output=True, text=True,
                       timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = m.logits(toks)
    got = np.concatenate([np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, 180) for i in (0, 2)])
    assert not (tmp_path / "1.f32").exists()
    assert error(got, want[[3, 39, 49]]) < LIMIT[F32 if dtype == "float32" else BF16]


def test_trace_refuses_a_dtype_the_family_lacks(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps(dict(vocab_size=64, hidden_size=64, num_hidden_layers=1,
                                                          num_attention_heads=1, intermediate_size=64)))
    assert trace_main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"]) == EXIT_DTYPE


@pytest.mark.parametrize("device", DEVICES)
def test_mixed_steps_of_the_existing_family(device):
    """The step function is the engine's, not one design's: Mistral-style models run it too."""
    from copilot_for_consensus_amd.runtime.trace import TraceSession
    cfg = registry.get_config("tiny")
    g = registry.build_model(registry.random_weights(cfg, device, seed=1))
    toks = torch.randint(3, 512, (90,), generator=torch.Generator().manual_seed(0)).tolist()

    def session():
        return TraceSession(LLMEngine(g, g.new_cache(16), use_graph=False, prefix_cache=False))
    want = torch.from_numpy(run(session(), "r", toks, [90]))
    s = session()
    got = [s.step([("r", toks[:50], list(range(50))), ("q", toks[:3], [])])]
    got.append(s.step([("q", toks[3:4], []), ("r", toks[50:80], list(range(30)))]))
    for i in range(80, 90):
        got.append(s.step([("r", toks[i:i + 1], [0]), ("q", toks[i:i + 1], [])]))
    assert error(np.concatenate(got), want) < 5e-2
