"""Kugilix models on the device against the plain statement (kugilix_plain.py): whole prompts with the residual
stream behind every layer run, decoding through the caches, prompts cut into portions, requests one after the other,
rings that wrap, and greedy generation through the engine and the command line."""
import json
import os
import subprocess

import numpy as np
import pytest

import kugilix_model as km
import kugilix_plain as plain

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# spread-relative: bfloat16 rounding of a few layers, binary32 rounding
LIMIT = {"bfloat16": 0.03, "float32": 2e-5}
NAMES = sorted(km.configs())
_cache = {}


def setup(tmp_path_factory, name):
    """(cfg, weights, folder, tokens, logits of every position, residual streams) of a configuration"""
    if name not in _cache:
        cfg = km.configs()[name]
        w = km.weights(cfg, 11 + NAMES.index(name))
        folder = str(tmp_path_factory.mktemp("kugilix_" + name))
        km.write(folder, cfg, w)
        tokens = np.random.default_rng(5).integers(0, cfg["vocab"], 211).tolist()
        taps = []
        logits = plain.forward(cfg, w, tokens, taps)
        _cache[name] = (cfg, w, folder, tokens, logits, np.stack(taps))
    return _cache[name]


@pytest.fixture(params=[(n, d) for n in NAMES for d in ("bfloat16", "float32")], ids=lambda p: "-".join(p))
def case(request, awq, torch_gpu, tmp_path_factory):
    name, dtype = request.param
    cfg, w, folder, tokens, logits, taps = setup(tmp_path_factory, name)
    print("kugilix", name, dtype, flush=True)
    eng = awq.open_model(folder, dtype=dtype, max_positions=400)
    yield eng, cfg, tokens, logits, taps, LIMIT[dtype]
    eng.close()


def test_whole_prompt_and_every_layer(case):
    eng, cfg, tokens, logits, taps, limit = case
    assert eng.architecture == "Kugilix" and eng.vocab_size == cfg["vocab"] and eng.hidden_size == cfg["width"]
    got = eng.forward(tokens, range(len(tokens)))
    assert km.rms_error(got, logits) < limit
    eng.set_layer_tap(True)
    eng.reset()
    eng.forward(tokens)
    got = eng.read_layer_tap().reshape(taps.shape)
    for i in range(len(taps)):
        assert km.rms_error(got[i], taps[i]) < limit, "layer run %d" % i
    # the same position by position (the one-token kernels)
    eng.reset()
    for t in range(12):
        eng.forward(tokens[t:t + 1])
        got = eng.read_layer_tap().reshape(len(taps), cfg["width"])
        for i in range(len(taps)):
            assert km.rms_error(got[i], taps[i][t]) < limit, "layer run %d, token %d" % (i, t)


def test_decoding_agrees_with_the_prompt(case):
    eng, cfg, tokens, logits, taps, limit = case
    for cut in (0, 1, 40, 130):
        eng.reset()
        if cut:
            eng.forward(tokens[:cut])
        got = np.concatenate([eng.forward([t], [0]) for t in tokens[cut:]])
        assert km.rms_error(got, logits[cut:]) < limit, "from token %d" % cut


@pytest.mark.parametrize("sizes", [[2], [3, 2], [7, 1, 20], [64], [63, 65, 2], [17, 128]], ids=str)
def test_portions(case, sizes):
    eng, cfg, tokens, logits, taps, limit = case
    eng.reset()
    got, at, i = [], 0, 0
    while at < len(tokens):
        n = min(sizes[i % len(sizes)], len(tokens) - at)
        got.append(eng.forward(tokens[at:at + n], range(n)))
        at, i = at + n, i + 1
    assert km.rms_error(np.concatenate(got), logits) < limit


def test_requests_one_after_the_other(case, awq):
    """what an earlier request left in caches, rings and states does not show in a later one"""
    eng, cfg, tokens, logits, taps, limit = case
    rng = np.random.default_rng(1)
    for n in (3, 150, 1, 70, 2, 211):
        eng.reset()
        eng.forward(rng.integers(0, cfg["vocab"], int(rng.integers(1, 300))).tolist())
        eng.reset()
        got = eng.forward(tokens[:n], range(n))
        assert km.rms_error(got, logits[:n]) < limit
        if n < 211:
            assert km.rms_error(eng.forward(tokens[n:n + 1], [0]), logits[n:n + 1]) < limit


def test_graphs_and_eager_steps_give_the_same(case):
    eng, cfg, tokens, logits, taps, limit = case
    eng.reset()
    eng.prefill(tokens[:50])
    a = [eng.decode(1)[0], *eng.decode(9), *eng.decode(30)]
    la = eng.read_logits_f32()
    eng.set_graph_mode(False)
    eng.reset()
    eng.prefill(tokens[:50])
    b = eng.decode(40)
    assert a == b and np.array_equal(la, eng.read_logits_f32())
    # captured steps again, after eager work
    eng.set_graph_mode(True)
    eng.reset()
    eng.prefill(tokens[:50])
    assert eng.decode(40) == b


def test_greedy_generation(case):
    """every generated token is the plain statement's choice, up to ties within rounding"""
    eng, cfg, tokens, logits, taps, limit = case
    w = _cache[[n for n in NAMES if km.configs()[n] == cfg][0]][1]
    prompt = tokens[:37]
    for batched in (True, False):
        eng.set_prefill_mode(batched)
        out = eng.generateResponse(prompt, 130)
        assert len(out) == 130
        z = plain.forward(cfg, w, prompt + out[:-1])[len(prompt) - 1:]
        short = z.max(axis=1) - z[np.arange(len(out)), out]
        assert short.max() <= 6 * limit * np.std(z)
        assert np.mean(short == 0) > (0.85 if limit > 1e-3 else 0.98)
    assert eng.generateResponse(prompt, 5) == out[:5]


def test_long_sequence_in_wrapping_rings(awq, torch_gpu, tmp_path):
    """more positions than a ring holds: a window behind one pass of 2048"""
    cfg = km.model(32, 64, [km.attention(2, 1, 16, 8, 9, ff=32), km.lightning(1, 8, 8, [0.99])], groups=2, taps=2)
    w = km.weights(cfg, 3)
    km.write(str(tmp_path), cfg, w)
    tokens = np.random.default_rng(9).integers(0, cfg["vocab"], 4400).tolist()
    ref = plain.forward(cfg, w, tokens)
    limits = {"bfloat16": 0.08, "float32": LIMIT["float32"]}  # the worst of 4400 rows of 64 logits
    for dtype in ("bfloat16", "float32"):
        eng = awq.open_model(str(tmp_path), dtype=dtype, max_positions=5000)
        got, at = [], 0
        for n in (2047, 100, 2, 1, 1, 1, 1900, 130, 2):
            got.append(eng.forward(tokens[at:at + n], range(n)))
            at += n
        while at < len(tokens):
            got.append(eng.forward(tokens[at:at + 1], [0]))
            at += 1
        assert km.rms_error(np.concatenate(got), ref) < limits[dtype]
        # one call, cut into passes by the engine
        eng.reset()
        assert km.rms_error(eng.forward(tokens, range(len(tokens))), ref) < limits[dtype]
        eng.close()


def test_float32_tensors_and_extra_keys(awq, torch_gpu, tmp_path):
    cfg = km.model(48, 96, [km.attention(2, 2, 24, 16, 7, ff=40)], groups=3)
    cfg["layers"][0]["mixer"]["unused"] = {"size": 3}
    w = km.weights(cfg, 4)
    w["l0.mix.q"] = (w["l0.mix.q"] * np.float32(1.0001)).astype(np.float32)  # no longer bfloat16 values
    km.write(str(tmp_path), cfg, w, f32_names=("l0.mix.q", "l0.norm1", "embed"))
    tokens = list(range(30))
    eng = awq.open_model(str(tmp_path), dtype="float32", max_positions=64)
    assert km.rms_error(eng.forward(tokens, range(30)), plain.forward(cfg, w, tokens)) < LIMIT["float32"]
    with pytest.raises(awq.AwqError):
        eng.forward([0] * 35)             # does not fit max_positions
    with pytest.raises(awq.AwqError):
        eng.forward([cfg["vocab"]])       # no such token
    with pytest.raises(awq.AwqError):
        eng.forward([1, 2], [1, 0])       # places must ascend
    eng.reset()
    with pytest.raises(awq.AwqError):
        eng.decode(1)                     # an empty sequence has nothing to continue
    eng.close()


def test_command_line_and_trace_runner(awq, torch_gpu, tmp_path):
    cfg = km.model(64, 80, [km.attention(4, 2, 16, 16, 6, ff=64), km.lightning(2, 16, 24, [0.6, 0.95], ff=64)], taps=4)
    w = km.weights(cfg, 8)
    folder = str(tmp_path / "m")
    km.write(folder, cfg, w)
    pkg = os.path.join(ROOT, "cuda-kernel-qwen3-8b-awq_amd")
    run = subprocess.run([os.path.join(pkg, "qwen3_awq_infer"), folder, "--prompt", "3,1,4,1,5", "--new", "12", "--dtype", "float32"],
                         capture_output=True, text=True, timeout=100)
    assert run.returncode == 0, run.stderr
    ids = [int(t) for t in run.stdout.split(":")[1].split()]
    want, gap = plain.generate(cfg, w, [3, 1, 4, 1, 5], 12)
    assert gap > 1e-4 and ids == want
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": [3, 1, 4], "want": [0, 2]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [1, 5], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": [9], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": [7, 7], "want": [1]}], "end": ["b"]}]
    for dtype in ("bfloat16", "float32"):
        out = tmp_path / dtype
        out.mkdir()
        run = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(out),
                              "--max-tokens", "16"], input="".join(json.dumps(s) + "\n" for s in steps),
                             capture_output=True, text=True, timeout=100)
        assert run.returncode == 0, run.stderr
        assert run.stdout.split("\n")[:4] == ["done %d" % i for i in range(4)]
        za, zb = plain.forward(cfg, w, [3, 1, 4, 1, 5, 9]), plain.forward(cfg, w, [7, 7])
        read = lambda n: np.fromfile(str(out / ("%d.f32" % n)), dtype="<f4").reshape(-1, cfg["vocab"])
        assert km.rms_error(read(0), za[[0, 2]]) < LIMIT[dtype]
        assert not (out / "1.f32").exists()
        assert km.rms_error(read(2), za[[5]]) < LIMIT[dtype]
        assert km.rms_error(read(3), zb[[1]]) < LIMIT[dtype]
