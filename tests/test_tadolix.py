"""The Tadolix decoder through the framework's loader, cache, state slots, step, engines and command line."""
import json
import os
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import tadolix_oracle as oracle
from copilot_for_consensus_amd.models import registry
from copilot_for_consensus_amd.models.tadolix import TadolixWeights, config_from_json
from copilot_for_consensus_amd.runtime.continuous import ContinuousEngine
from copilot_for_consensus_amd.runtime.engine import LLMEngine
from copilot_for_consensus_amd.runtime.trace import open_session
from tadolix_models import CONFIGS, Model, config, error, lru, par

ROOT = Path(__file__).resolve().parent.parent
DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F32, BF16 = torch.float32, torch.bfloat16
# relative to the logits' spread
LIMIT = {F32: 5e-5, BF16: 6e-2}
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


def run(sess, rid, toks, cuts):
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
    m = model(name)
    toks = m.tokens(171 if name == "wide" else 101)
    want = m.logits(toks)
    sess = m.session(device, dtype)
    for cuts in ([171], [64, 1], [1], [2], [3, 31, 2, 32, 2, 29, 1], [17, 16, 15, 1, 33, 2]):
        if name == "wide" and device == "cpu" and cuts[0] in (1, 2):
            continue                                       # slow here, and the others decode and cut as well
        got = run(sess, "r", toks, cuts)
        sess.end("r")
        assert error(got, want) < LIMIT[dtype], (cuts, error(got, want))
    assert sess.engine.kv.pool.num_free() == 64 and sess.engine.kv.states.num_free() == 4


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_prompts_over_many_segments(device, dtype):
    """Prompts of several segments of both recurrences, tiles of the convolutions and key tiles."""
    m = model("packed")
    toks = m.tokens(450)
    want = m.logits(toks)
    for cuts in ([450], [129, 130, 191], [400, 2, 48]):
        assert error(run(m.session(device, dtype), "r", toks, cuts), want) < LIMIT[dtype], cuts


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("n", [1, 2, 3, 6])
def test_first_tokens(device, n):
    """What lies before a sequence is zeros, for convolutions and states, whatever the slot held."""
    m = model("uneven")
    want, sess = m.logits(m.tokens(n)), m.session(device)
    run(sess, "used", m.tokens(9, seed=5), [9])            # leaves its state in the slot the next one takes
    sess.end("used")
    for cuts in ([n], [1], [2]):
        assert error(run(sess, "r", m.tokens(n), cuts), want) < LIMIT[F32]
        sess.end("r")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", ["uneven", "packed", "wide"])
def test_mixed_batches_equal_each_request_alone(name, dtype, device):
    """Portions beside single tokens; requests admitted, left out for a step, ended, and their blocks and state
    slots taken by others in a pool that holds no more than the live ones."""
    m = model(name)
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
        assert error(np.concatenate(got[r]), want[r]) < LIMIT[dtype], r


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


# ------------------------------------------------------------------ what a token reaches
def changed(m, toks, p):
    """The prompt with another token at p, and the plain model's logits of it."""
    t2 = list(toks)
    t2[p] = (t2[p] + 57) % m.cfg.vocab_size
    return t2, m.logits(t2)


def attention_only(size, **kw):
    """One layer whose attention alone carries a token to later ones."""
    m = Model(config([par(heads=2, kv_heads=1, dim=32, vdim=32, scale=0.05, size=size, width=8, ff=None, **kw)], taps=1), seed=2)
    m.tensors["l0.mix.right.o"].zero_()
    return m


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size", [37, 64, 1])
def test_chunk_edges_decide(device, size):
    """Even scores: a changed token moves the logits up to the last row of its chunk and not of the next chunk's rows; in
    prompts, in portions that start and end at the edge, and decoded."""
    m = attention_only(size)
    toks = m.tokens(130)
    want = m.logits(toks)
    for p in sorted({0, size - 1, size, size + 1, 2 * size - 1} | ({63, 64} if size > 1 else set())):
        t2, w2 = changed(m, toks, p)
        moved = (w2 - want).abs().amax(-1) / want.std()
        edge = (p // size + 1) * size
        assert moved[min(edge, 130) - 1] > 1e-3 and not moved[edge:].any(), p          # it does show
        for cuts in ([130], [edge - 1 or 1, 1], [edge, 2], [max(1, edge - 2), 3, 1]):
            got = run(m.session(device), "r", t2, cuts)
            assert error(got, w2) < LIMIT[F32], (p, cuts)
            assert not ((torch.from_numpy(got)[edge:] - want[edge:]).abs() > 1e-4).any(), (p, cuts)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_a_distance_stands_out(device, dtype):
    """One row of the distance table far above the others: every token reads those at its distances and hardly another,
    at both ends of the row."""
    for row in (0, 3, 4, 6, 9):                          # own distances, then runs of them, then all from 81 on
        m = attention_only(200, far=100, buckets=10)
        m.tensors["l0.mix.left.rel"].fill_(-3.0)
        m.tensors["l0.mix.left.rel"][row] = 9.0
        toks = m.tokens(260)
        want = m.logits(toks)
        starts = [n for n in range(200) if oracle.bucket(n, 10, 100) == row]
        for p in (5, 64):
            t2, w2 = changed(m, toks, p)
            moved, last = (w2 - want).abs().amax(-1) / want.std(), min(starts[-1], 199 - p)
            assert moved[p + starts[0]] > 2e-3 and moved[p + last] > 5e-4, (row, p)
            assert p + last == 199 or moved[p + last + 1] < 0.1 * moved[p + last], (row, p)
            for cuts in ([260], [p + starts[0], 1, 1, 200], [150, 1]):
                assert error(run(m.session(device, dtype), "r", t2, cuts), w2) < LIMIT[dtype], (row, p, cuts)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_a_far_key_stands_out(device, dtype):
    """One score far above hundreds of others in the same chunk: whoever misses the key or its page gives other logits; and
    the cap holds it down."""
    for cap in (40.0, 3.0):
        m = Model(config([par(heads=2, kv_heads=1, dim=32, vdim=32, scale=0.4, cap=cap, far=50, size=480, width=8, ff=None)], width=64, taps=1,
                         scale=1.0), seed=7)
        e = m.tensors["embed"]                               # every query looks along coordinate 0 for keys along coordinate 1
        e[:, 0], e[:, 1], e[7, 1] = 6.0, 0.0, 24.0
        q, k = m.tensors["l0.mix.left.q"], m.tensors["l0.mix.left.k"]
        for w, dims, at in ((q, (0, 32), 0), (k, (0,), 1)):
            w *= 0.2
            for d in dims:
                w[d, at] = 2.0
        for name in ("l0.canon1", "l0.norm1", "l0.mix.right.o"):
            m.tensors[name].zero_()
        toks = [t if t != 7 else 8 for t in m.tokens(500)]
        for at in (0, 31, 100, 131):
            t2 = list(toks)
            t2[at] = 7
            want = m.logits(t2)
            moved = ((want - m.logits(toks)).abs().amax(-1) / want.std())
            assert moved[400:480].median() > (0.05 if cap > 10 else 0.005) and not moved[480:].any()      # it does show, far on
            for cuts in ([500], [470, 1], [64, 1, 2, 100, 33, 300]):
                assert error(run(m.session(device, dtype), "r", t2, cuts), want) < LIMIT[dtype], (at, cuts)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["gru", "lru"])
def test_a_far_token_lives_in_the_state(device, kind):
    """Slow gates: the first and a chunk-border token move the logits hundreds of tokens later, as they move
    the plain model's."""
    layer = par(width=64, size=2, ff=None) if kind == "gru" else lru(width=64, blocks=2)
    m = Model(config([layer] * 2, loop=(0, 2, 2)), seed=3)
    for i in (0, 1):
        if kind == "gru":
            m.tensors[f"l{i}.mix.right.z.b"].fill_(-5.5)
            m.tensors[f"l{i}.mix.right.z"] *= 0.1
            m.tensors[f"l{i}.mix.left.o"].zero_()
        else:
            m.tensors[f"l{i}.mix.lam"].fill_(-7.0)
    toks = m.tokens(300)
    want = m.logits(toks)
    for p in (0, 63, 64, 127, 128):
        t2, w2 = changed(m, toks, p)
        assert (w2 - want)[299].abs().max() / want.std() > 1e-3, p
        for cuts in ([300], [290, 1], [7, 100, 2, 150, 1]):
            assert error(run(m.session(device), "r", t2, cuts), w2) < LIMIT[F32], (p, cuts)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("taps,conv", [(7, 2), (2, 7), (40, 1)])
def test_convolutions_reach_back_over_portions(device, taps, conv):
    """Many taps ahead of the mixer and inside it: every cut of a prompt, down to portions shorter than the taps."""
    m = Model(config([lru(conv=conv), par(size=5)], taps=taps), seed=5)
    toks = m.tokens(90)
    want = m.logits(toks)
    for n in range(1, 10):
        assert error(run(m.session(device), "r", toks, [n, 2, 1, n, 31, 33, 1]), want) < LIMIT[F32], n


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(device):
    for dtype in (F32, BF16):
        m = model("packed")
        toks = m.tokens(230)
        assert error(run(m.session(device, dtype), "r", toks, [4, 1]), m.logits(toks)) < LIMIT[dtype]


@pytest.mark.parametrize("device", DEVICES)
def test_far_positions(device):
    """Sinusoids tens of thousands of tokens on keep their digits (against 64-bit angles)."""
    from copilot_for_consensus_amd.ops import stream as S
    for W in (64, 65):
        pos = torch.tensor([0, 1, 4095, 70000, 1048575], dtype=torch.int32)
        got = S.embed_f32(torch.zeros(3, W, device=device), torch.zeros(5, dtype=torch.int32, device=device), torch.empty(5, W, device=device),
                          2.0, pos.to(device), S.sinusoid_turns(W, 10000.0, device))
        e = torch.arange(W)
        a = pos[:, None].double() * 10000.0 ** (-2.0 * (e // 2).double() / W)
        assert float((got.cpu() - torch.where(e % 2 == 0, a.sin(), a.cos())).abs().max()) < 1e-6


def test_stream_after_every_layer():
    """The plain model's and the framework's streams, layer run by layer run."""
    m = model("uneven")
    toks = m.tokens(33)
    after = oracle.forward(m.json, m.tensors, toks)[1]
    runs = m.cfg.runs
    assert runs == (0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4, 5) and after.shape[0] == 12
    for n in range(1, len(runs) + 1):
        sub = Model(dict(m.json, layers=[m.json["layers"][i] for i in runs[:n]], loop=None))
        sub.tensors = dict(m.tensors)
        for at, i in enumerate(runs[:n]):
            sub.tensors |= {f"l{at}." + k[len(f"l{i}."):]: v for k, v in m.tensors.items() if k.startswith(f"l{i}.")}
        x = oracle.norm(after[n - 1], m.tensors["final.norm"].float(), 3e-5) @ m.tensors["head"].float().T
        assert error(run(sub.session("cpu"), "r", toks, [33]), x) < LIMIT[F32], n


# ------------------------------------------------------------------ loading and registry
@pytest.mark.parametrize("device", DEVICES)
def test_checkpoint_through_the_registry(tmp_path, device):
    m = model("uneven")
    d = m.save(tmp_path / "ckpt")
    cfg = registry.load_config_json(d / "config.json")
    assert cfg.specs == m.cfg.specs and cfg.norm_eps == 3e-5 and cfg.loop == (1, 4, 3) and cfg.streams == 2
    assert registry.family_of(cfg).name == "Tadolix"
    toks = m.tokens(37)
    sess = open_session(d, "float32", 64, device=device)
    kv = sess.engine.kv
    assert kv.num_blocks == 2 and kv.states.n == 4 and sess.engine.prefix_cache is None
    # every pass through a layer has a cache and a state of its own
    assert [h is not None for h in kv.heads] == [True, False, False, True] + [False, False, True] * 2 + [True, False]
    assert len({t.data_ptr() for t in kv.recur}) == 12 and all(t.shape[1:] == (2, 104) for t in kv.inputs)
    assert error(run(sess, "r", toks, [20, 17]), m.logits(toks)) < LIMIT[F32]


def test_loader_refuses_what_does_not_fit(tmp_path):
    m = model("uneven")
    d = m.save(tmp_path / "ckpt")
    with pytest.raises(ValueError, match="embed"):
        TadolixWeights.from_safetensors(config_from_json(dict(m.json, vocab=181)), d, "cpu")
    with pytest.raises(KeyError, match="missing"):
        TadolixWeights.from_safetensors(config_from_json(dict(m.json, layers=m.json["layers"] + [lru()])), d, "cpu")
    for bad in (dict(par(), type="ring"), dict(par(), mlp={"kind": "moe"})):
        with pytest.raises(NotImplementedError):
            config_from_json(config([bad]))
    for bad in (config([par()], streams=17), config([par()], taps=0), config([par()], loop=(0, 2, 2)), config([lru(width=10, blocks=3)]),
                config([par(heads=3, kv_heads=2)])):
        with pytest.raises(ValueError):
            config_from_json(bad)
    with pytest.raises(ValueError, match="distance bias"):
        registry.build_model(TadolixWeights._build(config_from_json(config([par(far=5, buckets=10)])), Model(config([par()])).tensors.get,
                                                   "cpu", 0, 1, F32))
    assert registry.get_config("tiny-tadolix").layers == 4


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
    than requests: the plain model's tokens."""
    m = Model(config([par(dim=24, size=19, ff=40), lru(width=48), lru(width=32, blocks=2, conv=5, ff=33)], width=64, loop=(0, 2, 2)), seed=6)
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
    m = Model(config([par(ff=40), lru()], vocab=512, width=64), seed=5)
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
    s = HipLLMSummarizer(model="tiny-tadolix", device="cpu", kv_cache_tokens=2048, ignore_eos=True, max_new_tokens=4)
    assert s.model == "tiny-tadolix"
    res = s.engine.generate([[1, 2, 3]], 4, ignore_eos=True)
    assert len(res.tokens[0]) == 4
    d = model("packed").save(tmp_path / "mine")
    s = HipLLMSummarizer(checkpoint_dir=str(d), device="cpu", kv_cache_tokens=512, ignore_eos=True, max_new_tokens=4)
    assert s.model == "mine" and s.cfg.vocab_size == 320


# ------------------------------------------------------------------ tensor parallel
def _tp_model():
    return Model(config([par(ff=48), lru(width=64, blocks=4, ff=24), par(heads=2, size=9, width=6, ff=None)], loop=(0, 2, 2)), seed=8)


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
    m = model("packed")
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
    got = np.concatenate([np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, 320) for i in (0, 2)])
    assert not (tmp_path / "1.f32").exists()
    assert error(got, m.logits(toks)[[3, 39, 49]]) < LIMIT[F32 if dtype == "float32" else BF16]
