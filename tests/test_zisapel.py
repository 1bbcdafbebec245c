"""The Zisapel decoder through the framework's loader, cache, state slots, step, engines and command line."""
import json
import os
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

from copilot_for_consensus_amd.models import registry
from copilot_for_consensus_amd.models.zisapel import ZisapelWeights, config_from_json
from copilot_for_consensus_amd.runtime.continuous import ContinuousEngine
from copilot_for_consensus_amd.runtime.engine import LLMEngine
from copilot_for_consensus_amd.runtime.trace import open_session
from zisapel_models import CONFIGS, Model, attn, config, dense, error, moe, wkv

ROOT = Path(__file__).resolve().parent.parent
DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F32, BF16 = torch.float32, torch.bfloat16
# relative to the logits' spread
LIMIT = {F32: 5e-5, BF16: 8e-2}
# seven uneven layers carry bf16 rounding further than the others do
LOOSE = {"uneven": 6.0}
_models: dict = {}


@pytest.fixture(autouse=True)
def one_thread():
    """The CPU cases are many small operations: threads only get in each other's way."""
    n = torch.get_num_threads()
    torch.set_num_threads(1)
    yield
    torch.set_num_threads(n)


def model(name, dtype=F32) -> Model:
    """In bf16 a choice of experts that rounding turns would stay in the state for all that follows: steady choices."""
    key = (name, dtype == BF16)
    if key not in _models:
        _models[key] = Model(name, steady=dtype == BF16)
    return _models[key]


def run(sess, rid, toks, cuts):
    """Feed toks to request rid in portions of the given sizes (the last repeats); all logits."""
    out, at, i = [], 0, 0
    while at < len(toks):
        n = min(cuts[min(i, len(cuts) - 1)], len(toks) - at)
        out.append(sess.step([(rid, toks[at:at + n], list(range(n)))]))
        at, i = at + n, i + 1
    return np.concatenate(out)


def row_errors(got, want):
    d = torch.as_tensor(got, dtype=torch.float32) - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.std()


def fits(got, want, dtype, loose=1.0):
    """Every row in fp32; in bf16 all but a tenth (a small branch's norm magnifies what is left of its rounding)."""
    e = row_errors(got, want)
    return float(e.max() if dtype == F32 else e.quantile(0.9)) < LIMIT[dtype] * loose


# ------------------------------------------------------------------ whole prompts, portions, decoding
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_portions_and_decoding(name, dtype, device):
    m, toks = model(name, dtype), model(name).tokens(101)
    want = m.logits(toks)
    sess = m.session(device, dtype)
    for cuts in ([101], [64, 1], [1], [2], [3, 31, 2, 32, 2, 29, 1], [17, 16, 15, 1, 33, 2]):
        got = run(sess, "r", toks, cuts)
        sess.end("r")
        assert fits(got, want, dtype, LOOSE.get(name, 1.0) if dtype == BF16 else 1.0), (cuts, row_errors(got, want))
    assert sess.engine.kv.pool.num_free() == 64 and sess.engine.kv.states.num_free() == 4


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("n", [1, 2, 3, 4])
def test_first_tokens(device, n):
    """What lies before a sequence is zeros: the shift looks two tokens back, in prompts and decoded."""
    m = model("uneven")
    want, sess = m.logits(m.tokens(n)), m.session(device)
    run(sess, "used", m.tokens(9, seed=5), [9])            # leaves its state in the slot the next one takes
    sess.end("used")
    for cuts in ([n], [1]):
        assert error(run(sess, "r", m.tokens(n), cuts), want) < LIMIT[F32]
        sess.end("r")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", ["uneven", "packed", "wide"])
def test_mixed_batches_equal_each_request_alone(name, dtype, device):
    """Portions beside single tokens; requests admitted, left out for a step, ended, and their blocks and state
    slots taken by others in a pool that holds no more than the live ones."""
    m = model(name, dtype)
    lens = {"a": 150, "b": 40, "c": 97, "d": 33, "e": 66, "f": 5}
    toks = {r: m.tokens(n, seed=i) for i, (r, n) in enumerate(lens.items())}
    want = {r: m.logits(t) for r, t in toks.items()}
    sess = m.session(device, dtype, blocks=13, sequences=3)
    at, live, queue, held = dict.fromkeys(lens, 0), [], list(lens), {}
    gen, got = np.random.default_rng(5), {r: [] for r in lens}
    while queue or live:
        while queue and len(live) < 3 and sum(held.values()) + -(-lens[queue[0]] // 32) <= 13:
            live.append(queue.pop(0))
            held[live[-1]] = -(-lens[live[-1]] // 32)
        step = []
        for r in live:
            n = min(int(gen.choice([0, 1, 1, 2, 3, 31, 32, 64])), lens[r] - at[r])
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
                del held[r]
    for r in lens:
        assert fits(np.concatenate(got[r]), want[r], dtype, LOOSE.get(name, 1.0) if dtype == BF16 else 1.0), r


@pytest.mark.parametrize("device", DEVICES)
def test_logits_do_not_depend_on_pages_slots_or_company(device):
    m = model("uneven")
    toks, other = m.tokens(70), m.tokens(45, seed=9)
    base = torch.from_numpy(run(m.session(device), "r", toks, [70]))
    sess = m.session(device, blocks=8)
    run(sess, "x", other, [45])                         # takes blocks and a slot first, leaves stale values behind
    sess.end("x")
    sess.step([("y", other[:40], [])])
    assert error(run(sess, "r", toks, [9, 2, 27, 1]), base) < 2e-5
    both = sess.step([("y", other[40:], []), ("z", toks[:33], [0, 32]), ("w", toks[:1], [0])])
    assert error(both, base[[0, 32, 0]]) < 2e-5


@pytest.mark.parametrize("device", DEVICES)
def test_window_edges_decide(device):
    """Even scores: a changed token moves the logits of the last row that sees it and not of the next one, in
    prompts and decoded.  Without shift and recurrence nothing else carries it."""
    size = 37
    m = Model(config([attn(heads=2, dim=32, rot_dim=8, vdim=32, kv_rank=64, scale=0.05, size=size, mlp=None)]), seed=2)
    m.tensors["l0.shift"].zero_()
    m.tensors["l0.mix.sink"].fill_(-4.0)
    toks = m.tokens(110)
    want = m.logits(toks)
    for p in (0, 31, 32, 63, 64):
        t2 = list(toks)
        t2[p] = (t2[p] + 57) % 180
        w2 = m.logits(t2)
        moved = (w2 - want).abs().amax(-1) / want.std()
        assert moved[p + size - 1] > 1e-3 and moved[p + size] == 0, p          # it does show
        for cuts in ([110], [p + size - 2 or 1, 1], [p + size, 2]):
            got = run(m.session(device), "r", t2, cuts)
            assert error(got, w2) < LIMIT[F32], (p, cuts)
            assert float((torch.from_numpy(got)[p + size:] - want[p + size:]).abs().max()) < 1e-4


@pytest.mark.parametrize("device", DEVICES)
def test_a_far_token_lives_in_the_state(device):
    """Slow decays: the first and a chunk-border token move the logits hundreds of tokens later, as they move
    the plain model's."""
    m = Model(config([wkv(heads=2, dim=32, mlp=None)] * 2), seed=3)
    for i in (0, 1):
        m.tensors[f"l{i}.mix.w0"].fill_(-7.0)
        m.tensors[f"l{i}.mix.w2"] *= 0.1
    toks = m.tokens(300)
    want = m.logits(toks)
    for p in (0, 15, 16, 255):
        t2 = list(toks)
        t2[p] = (t2[p] + 57) % 180
        w2 = m.logits(t2)
        assert (w2 - want)[299].abs().max() / want.std() > 1e-3, p
        for cuts in ([300], [290, 1], [7, 100, 2, 150, 1]):
            assert error(run(m.session(device), "r", t2, cuts), w2) < LIMIT[F32], (p, cuts)


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(device):
    for dtype in (F32, BF16):
        m = model("packed", dtype)
        toks = m.tokens(230)
        assert fits(run(m.session(device, dtype), "r", toks, [4, 1]), m.logits(toks), dtype)


@pytest.mark.gpu
def test_long_portions_expand_keys_and_values():
    """The pass chooses per-head keys and values for long portions; both ways give the plain model's logits."""
    m = model("wide")
    toks = m.tokens(500)
    want = m.logits(toks)
    g = m.build("cuda", BF16)
    assert "uk_full" in g.w.layers[0] and "uk_full" in g.w.layers[2]
    chosen = g._expand_pays
    assert not chosen([0, 1], [500], 128, 150) and chosen([0, 4000], [4000], 512, 2048)
    try:
        for force in (False, True):
            g._expand_pays = lambda cu, ctx, rv, window: force
            for cuts in ([500], [233, 2, 200, 65], [64, 1, 300]):
                got = run(m.session("cuda", BF16), "r", toks, cuts)
                assert float(row_errors(got, want).max()) < LIMIT[BF16], (force, cuts)
    finally:
        g._expand_pays = chosen


# ------------------------------------------------------------------ loading and registry
@pytest.mark.parametrize("device", DEVICES)
def test_checkpoint_through_the_registry(tmp_path, device):
    m = model("uneven")
    d = m.save(tmp_path / "ckpt")
    cfg = registry.load_config_json(d / "config.json")
    assert cfg.specs == m.cfg.specs and cfg.norm_eps == 3e-5 and cfg.logit_scale == 0.7
    assert cfg.specs[1].mixer.rank == 7                  # from the tensor's shape
    assert registry.family_of(cfg).name == "Zisapel"
    toks = m.tokens(37)
    sess = open_session(d, "float32", 64, device=device)
    assert sess.engine.kv.num_blocks == 2 and sess.engine.kv.states.n == 4 and sess.engine.prefix_cache is None
    assert error(run(sess, "r", toks, [20, 17]), m.logits(toks)) < LIMIT[F32]


def test_loader_refuses_what_does_not_fit(tmp_path):
    m = model("uneven")
    d = m.save(tmp_path / "ckpt")
    with pytest.raises(ValueError, match="embed"):
        ZisapelWeights.from_safetensors(config_from_json(dict(m.json, vocab=181)), d, "cpu")
    with pytest.raises(KeyError, match="missing"):
        ZisapelWeights.from_safetensors(config_from_json(dict(m.json, layers=m.json["layers"] + [wkv()])), d, "cpu")
    for bad in (dict(wkv(), type="ring"), dict(wkv(), mlp={"kind": "tree"})):
        with pytest.raises(NotImplementedError):
            config_from_json(config([bad]))
    no_rank = wkv()
    del no_rank["mixer"]["rank"]
    with pytest.raises(ValueError, match="rank"):
        config_from_json(config([no_rank]))
    assert registry.get_config("tiny-zisapel").layers == 4


def test_parameter_count():
    m = model("uneven")
    assert m.cfg.num_params() == sum(t.numel() for t in m.tensors.values())


# ------------------------------------------------------------------ state slots
def test_state_slots_run_out_and_come_back():
    m = Model(config([wkv(mlp=None)]), seed=1)
    g = m.build("cpu")
    eng = LLMEngine(g, g.new_cache(16, sequences=2))
    prompts = [m.tokens(5, seed=i) for i in range(3)]
    with pytest.raises(MemoryError):
        eng.generate(prompts, 2, ignore_eos=True)
    assert eng.kv.states.num_free() == 2 and eng.kv.pool.num_free() == 16
    assert len(eng.generate(prompts[:2], 2, ignore_eos=True).tokens) == 2
    assert eng.kv.states.num_free() == 2 and eng.prefix_cache is None


# ------------------------------------------------------------------ generation
def greedy(m, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(m.logits(toks)[-1].argmax()))
    return toks[len(prompt):]


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_both_engines(device):
    """LLMEngine (decode graph on the GPU, replayed and captured anew), then ContinuousEngine with fewer slots
    than requests: the plain model's tokens."""
    m = Model(config([wkv(heads=2, dim=24, mlp=dense(40)), attn(heads=2, size=19, mlp=moe(experts=8)), wkv(heads=3, mlp=None)],
                     width=64), seed=6)
    prompts = [m.tokens(75), m.tokens(1), m.tokens(103), m.tokens(31), m.tokens(66)]
    want = [greedy(m, p, 9) for p in prompts]
    g = m.build(device)
    eng = LLMEngine(g, g.new_cache(64, sequences=6), max_prefill_tokens=64)
    for _ in range(3):
        res = eng.generate(prompts, 9, ignore_eos=True)
        assert res.tokens == want
    if device == "cuda":
        assert eng.last_used_graph
    ce = ContinuousEngine(eng, max_slots=2, max_new_cap=16, max_prompt=128, steps_per_sync=4, max_wait_s=0.0)
    reqs = [ce.submit(p, 9) for p in prompts]
    ce.run()
    assert [r.tokens for r in reqs] == want
    ce.close()
    assert eng.kv.states.num_free() == 6


@pytest.mark.parametrize("device", DEVICES)
def test_stop_strings_and_sampling(device):
    """The engine's own stops and sampler over the family: a stopped row ends where its text does, its slot comes
    back; the same seed draws the same tokens."""
    from copilot_for_consensus_amd.runtime.stops import StopStringMatcher
    from test_stops import STOPS, _vocab_tok
    m = Model(config([wkv(heads=2, dim=16, mlp=dense(40)), attn(heads=2, mlp=None)], vocab=512, width=64), seed=5)
    g = m.build(device)
    eng = LLMEngine(g, g.new_cache(64, sequences=6))
    matcher = StopStringMatcher.for_tokenizer(_vocab_tok(512), STOPS)
    prompts = [m.tokens(20 + i, seed=i) for i in range(6)]
    full = eng.generate(prompts, 40, temperature=1.5, seed=11, ignore_eos=True).tokens
    assert eng.generate(prompts, 40, temperature=1.5, seed=11, ignore_eos=True).tokens == full
    res = eng.generate(prompts, 40, temperature=1.5, seed=11, ignore_eos=True, stop_strings=matcher).tokens
    cut = [matcher.match_tokens(t) for t in full]
    assert any(c is not None for c in cut)
    for whole, c, got in zip(full, cut, res):
        assert got == (whole if c is None else whole[:c + 1])
    assert eng.kv.states.num_free() == 6


@pytest.mark.gpu
def test_decode_graph_replays_equal_eager_steps():
    m = model("packed")
    g = m.build("cuda", BF16)
    prompts = [m.tokens(n, seed=n) for n in (40, 7, 64, 33, 5, 90)]
    a = LLMEngine(g, g.new_cache(64), use_graph=True)
    b = LLMEngine(g, g.new_cache(64), use_graph=False)
    want = b.generate(prompts, 24, ignore_eos=True).tokens
    for _ in range(3):
        assert a.generate(prompts, 24, ignore_eos=True).tokens == want
        torch.cuda.synchronize()


def test_summarizer_serves_the_family(tmp_path):
    from copilot_for_consensus_amd.summarization import HipLLMSummarizer
    s = HipLLMSummarizer(model="tiny-zisapel", device="cpu", kv_cache_tokens=2048, ignore_eos=True, max_new_tokens=4)
    assert s.model == "tiny-zisapel"
    res = s.engine.generate([[1, 2, 3]], 4, ignore_eos=True)
    assert len(res.tokens[0]) == 4
    d = model("packed").save(tmp_path / "mine")
    s = HipLLMSummarizer(checkpoint_dir=str(d), device="cpu", kv_cache_tokens=512, ignore_eos=True, max_new_tokens=4)
    assert s.model == "mine" and s.cfg.vocab_size == 256


# ------------------------------------------------------------------ tensor parallel
def _tp_model():
    return Model(config([wkv(heads=4, mlp=dense(48)), attn(heads=2, mlp=moe(ff=24, shared=40)), wkv(heads=2, mlp=None)]), seed=8)


def _tp_worker(rank, port, out):
    os.environ.update(MASTER_ADDR="127.0.0.1", MASTER_PORT=str(port), GLOO_SOCKET_IFNAME="lo")
    torch.distributed.init_process_group("gloo", rank=rank, world_size=2)
    m = _tp_model()
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
    m = _tp_model()
    assert json.loads((tmp_path / "t.json").read_text()) == [greedy(m, m.tokens(40), 6), greedy(m, m.tokens(3), 6)]


# ------------------------------------------------------------------ trace replay
@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_run_program(tmp_path, dtype):
    m = model("packed", BF16)
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
    got = np.concatenate([np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, 256) for i in (0, 2)])
    assert not (tmp_path / "1.f32").exists()
    assert error(got, m.logits(toks)[[3, 39, 49]]) < LIMIT[F32 if dtype == "float32" else BF16]
