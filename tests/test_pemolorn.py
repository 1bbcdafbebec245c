"""The Pemolorn decoder through the framework's loader, cache, state slots, step, engines and command line."""
import json
import os
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import pemolorn_oracle as oracle
from copilot_for_consensus_amd.models import registry
from copilot_for_consensus_amd.models.pemolorn import PemolornWeights, config_from_json
from copilot_for_consensus_amd.runtime.continuous import ContinuousEngine
from copilot_for_consensus_amd.runtime.engine import LLMEngine
from copilot_for_consensus_amd.runtime.trace import open_session
from pemolorn_models import CONFIGS, Model, attn, config, dense, error, moe, par

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


# ------------------------------------------------------------------ whole prompts, portions, decoding
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_portions_and_decoding(name, dtype, device):
    m = model(name, dtype)
    toks = m.tokens(171 if name == "wide" else 101)
    want = m.logits(toks)
    sess = m.session(device, dtype)
    for cuts in ([171], [64, 1], [1], [2], [3, 31, 2, 32, 2, 29, 1], [17, 16, 15, 1, 33, 2]):
        got = run(sess, "r", toks, cuts)
        sess.end("r")
        assert error(got, want) < LIMIT[dtype], (cuts, error(got, want))
    assert sess.engine.kv.pool.num_free() == 64 and sess.engine.kv.states.num_free() == 4


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


def changed(m, toks, p):
    """The prompt with another token at p, and the plain model's logits of it."""
    t2 = list(toks)
    t2[p] = (t2[p] + 57) % m.cfg.vocab_size
    return t2, m.logits(t2)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("keep", [0, 5])
def test_window_edges_and_kept_tokens_decide(device, keep):
    """Even scores: a changed token moves the logits of the last row whose window holds it and not of the next one,
    unless it is kept; in prompts and decoded."""
    size = 37
    m = Model(config([attn(heads=2, kv_heads=1, dim=32, vdim=32, scale=0.05, size=size, keep=keep, mlp=None)]), seed=2)
    m.tensors["l0.mix.sink"].fill_(-4.0)
    toks = m.tokens(110)
    want = m.logits(toks)
    for p in (0, 4, 5, 31, 32, 63, 64):
        t2, w2 = changed(m, toks, p)
        moved = (w2 - want).abs().amax(-1) / want.std()
        assert moved[p + size - 1] > 1e-3 and (moved[p + size] > 1e-3) == (p < keep), p          # it does show
        for cuts in ([110], [p + size - 2 or 1, 1], [p + size, 2]):
            got = run(m.session(device), "r", t2, cuts)
            assert error(got, w2) < LIMIT[F32], (p, cuts)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size,pool", [(20, 8), (33, 5), (7, 32), (16, 48)])
def test_pooled_blocks_decide(device, size, pool):
    """Even scores: a changed token shows while the window holds it, not between its leaving and its block's coming
    into sight, and again from there on; in prompts, decoded, and with blocks ended in another portion."""
    c = config([par(heads=2, kv_heads=2, dim=32, vdim=32, scale=0.05, size=size, pool=pool, conv=1, rot=0, width=8, mlp=None)])
    m = Model(c, seed=4)
    m.tensors["l0.mix.left.sink"].fill_(-4.0)
    m.tensors["l0.mix.right.o"].zero_()                  # the recurrence would carry it
    toks = m.tokens(160)
    want = m.logits(toks)
    for p in (0, pool - 1, pool, 3 * pool // 2, 2 * pool + 1):
        t2, w2 = changed(m, toks, p)
        moved = (w2 - want).abs().amax(-1) / want.std()
        seen = (p // pool + 1) * pool - 1 + size          # the first row that sees the block
        if seen >= 160:
            continue
        assert moved[p + size - 1] > 1e-4 and moved[seen] > 1e-4 and not moved[p + size:seen].any(), p
        for cuts in ([160], [max(1, p), 1], [p + 1, 2], [seen - 1, 1], [seen, 2]):
            got = run(m.session(device), "r", t2, cuts)
            assert error(got, w2) < LIMIT[F32], (p, cuts)
            assert not ((torch.from_numpy(got)[p + size:seen] - want[p + size:seen]).abs() > 1e-4).any(), (p, cuts)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_a_far_key_stands_out(device, dtype):
    """One score far above hundreds of others, under a kept token and under a pooled block: whoever misses the key, its
    block or its page gives other logits."""
    c = config([attn(heads=2, kv_heads=1, dim=32, vdim=32, scale=0.5, size=40, keep=3, mlp=None),
                par(heads=2, kv_heads=1, dim=32, vdim=32, scale=0.5, size=40, pool=8, conv=1, rot=0, width=8, mlp=None)], width=64)
    m = Model(c, seed=7)
    e = m.tensors["embed"]                               # every query looks along coordinate 0 for keys along coordinate 1
    e[:, 0], e[:, 1], e[7, 1] = 3.0, 0.0, 12.0
    for x in ("l0.mix.", "l1.mix.left."):
        q, k = m.tensors[x + "q"], m.tensors[x + "k"]
        for w, dims, at in ((q, (0, 32), 0), (k, (0,), 1)):
            w *= 0.3
            for d in dims:
                w[d, at] = 2.0
        m.tensors[x + "q.norm"][::32] = m.tensors[x + "k.norm"][0] = 1.0
    m.tensors["l1.mix.right.o"].zero_()
    toks = [t if t != 7 else 8 for t in m.tokens(500)]
    for at in (2, 100, 131):
        t2 = list(toks)
        for k in range(8 if at > 2 else 1):
            t2[at // 8 * 8 + k if at > 2 else at] = 7
        want = m.logits(t2)
        assert ((want - m.logits(toks))[400:].abs().amax(-1) / want.std()).median() > 0.05      # it does show, far on
        for cuts in ([500], [480, 1], [64, 1, 2, 100, 33, 300]):
            assert error(run(m.session(device, dtype), "r", t2, cuts), want) < LIMIT[dtype], (at, cuts)


@pytest.mark.parametrize("device", DEVICES)
def test_a_far_token_lives_in_the_state(device):
    """Slow gates: the first and a chunk-border token move the logits hundreds of tokens later, as they move
    the plain model's."""
    m = Model(config([par(width=64, size=2, mlp=None)] * 2), seed=3)
    for i in (0, 1):
        m.tensors[f"l{i}.mix.right.z.b"].fill_(-5.5)
        m.tensors[f"l{i}.mix.right.z"] *= 0.1
        m.tensors[f"l{i}.mix.left.o"].zero_()
    toks = m.tokens(300)
    want = m.logits(toks)
    for p in (0, 63, 64, 255):
        t2, w2 = changed(m, toks, p)
        assert (w2 - want)[299].abs().max() / want.std() > 1e-3, p
        for cuts in ([300], [290, 1], [7, 100, 2, 150, 1]):
            assert error(run(m.session(device), "r", t2, cuts), w2) < LIMIT[F32], (p, cuts)


@pytest.mark.parametrize("device", DEVICES)
def test_convolution_reaches_back_over_portions(device):
    """Seven taps: every cut of a prompt, down to portions shorter than the taps."""
    m = Model(config([par(conv=7, mlp=None)]), seed=5)
    toks = m.tokens(40)
    want = m.logits(toks)
    for n in range(1, 10):
        assert error(run(m.session(device), "r", toks, [n, 2, 1, n]), want) < LIMIT[F32], n


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(device):
    for dtype in (F32, BF16):
        m = model("packed", dtype)
        toks = m.tokens(230)
        assert error(run(m.session(device, dtype), "r", toks, [4, 1]), m.logits(toks)) < LIMIT[dtype]


def test_stream_after_every_layer():
    """The plain model's and the framework's streams, layer by layer."""
    m = model("uneven")
    toks = m.tokens(33)
    after = oracle.forward(m.json, m.tensors, toks)[1]
    for n in range(1, len(m.json["layers"]) + 1):
        sub = Model(dict(m.json, layers=m.json["layers"][:n]))
        sub.tensors = {k: m.tensors[k] for k in sub.tensors}
        x = oracle.scalar_norm(after[n - 1], m.tensors["final.norm"].float(), 3e-5) @ m.tensors["head"].float().T
        assert error(run(sub.session("cpu"), "r", toks, [33]), x) < LIMIT[F32], n


# ------------------------------------------------------------------ loading and registry
@pytest.mark.parametrize("device", DEVICES)
def test_checkpoint_through_the_registry(tmp_path, device):
    m = model("uneven")
    d = m.save(tmp_path / "ckpt")
    cfg = registry.load_config_json(d / "config.json")
    assert cfg.specs == m.cfg.specs and cfg.norm_eps == 3e-5
    assert registry.family_of(cfg).name == "Pemolorn"
    toks = m.tokens(37)
    sess = open_session(d, "float32", 64, device=device)
    kv = sess.engine.kv
    assert kv.num_blocks == 2 and kv.states.n == 4 and sess.engine.prefix_cache is None
    assert kv.heads[3] is kv.heads[2] and kv.heads[7] is kv.heads[2] and kv.heads[5] is kv.heads[0]
    assert error(run(sess, "r", toks, [20, 17]), m.logits(toks)) < LIMIT[F32]


def test_loader_refuses_what_does_not_fit(tmp_path):
    m = model("uneven")
    d = m.save(tmp_path / "ckpt")
    with pytest.raises(ValueError, match="embed"):
        PemolornWeights.from_safetensors(config_from_json(dict(m.json, vocab=181)), d, "cpu")
    with pytest.raises(KeyError, match="missing"):
        PemolornWeights.from_safetensors(config_from_json(dict(m.json, layers=m.json["layers"] + [attn()])), d, "cpu")
    for bad in (dict(attn(), type="ring"), dict(attn(), mlp={"kind": "tree"})):
        with pytest.raises(NotImplementedError):
            config_from_json(config([bad]))
    for layers in ([attn(kv_from=0)], [attn(), attn(kv_from=1)], [par(), attn(kv_from=0)], [attn(), attn(kv_heads=1, kv_from=0)],
                   [attn(), attn(kv_from=0), attn(kv_from=1)]):
        with pytest.raises(ValueError, match="layer"):
            config_from_json(config(layers))
    assert registry.get_config("tiny-pemolorn").layers == 4


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
    m = Model(config([par(dim=24, size=19, mlp=dense(40)), attn(size=25, mlp=moe(experts=8)), attn(size=9, kv_from=1, mlp=None)], width=64),
              seed=6)
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
    m = Model(config([par(mlp=dense(40)), attn(mlp=None)], vocab=512, width=64), seed=5)
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
    m = model("packed", BF16)
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
    s = HipLLMSummarizer(model="tiny-pemolorn", device="cpu", kv_cache_tokens=2048, ignore_eos=True, max_new_tokens=4)
    assert s.model == "tiny-pemolorn"
    res = s.engine.generate([[1, 2, 3]], 4, ignore_eos=True)
    assert len(res.tokens[0]) == 4
    d = model("packed").save(tmp_path / "mine")
    s = HipLLMSummarizer(checkpoint_dir=str(d), device="cpu", kv_cache_tokens=512, ignore_eos=True, max_new_tokens=4)
    assert s.model == "mine" and s.cfg.vocab_size == 320


# ------------------------------------------------------------------ tensor parallel
def _tp_model():
    return Model(config([par(mlp=dense(48)), attn(mlp=moe(ff=24)), attn(size=9, kv_from=1, mlp=None)]), seed=8)


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
    got = np.concatenate([np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, 320) for i in (0, 2)])
    assert not (tmp_path / "1.f32").exists()
    assert error(got, m.logits(toks)[[3, 39, 49]]) < LIMIT[F32 if dtype == "float32" else BF16]
