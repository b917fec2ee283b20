"""Tudasun models on the device against the plain statement (tudasun_plain.py): whole prompts with the residual stream
behind every layer, decoding through caches and states, prompts cut into portions, requests one after the other, sequences
of several passes, and greedy generation through the engine and the command line."""
import json
import os
import subprocess

import numpy as np
import pytest

import kugilix_model as km
import tudasun_model as tm
import tudasun_plain as plain

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# spread-relative: bfloat16 rounding of a few layers with two norms and a gate each, binary32 rounding
LIMIT = {"bfloat16": 0.06, "float32": 5e-5}
# In bfloat16 a token whose router is all but undecided between two outputs may take the other one: its rows are left out,
# and a few rows near it (whose states and keys have seen it) may be over the limit.
CLOSE, SHARE = 0.015, {"bfloat16": 0.03, "float32": 0.0}
NAMES = sorted(tm.configs())
LENGTH = 331
_cache = {}


def margin(z, correction, top, groups):
    """how far the choice of plain.choose is from another one"""
    s = np.exp(z - z.max())
    choice = s / s.sum() + correction
    m = np.inf
    if groups:
        g = choice.reshape(groups["count"], -1)
        best = np.sort(g.max(axis=1))[::-1]
        if groups["keep"] < groups["count"]:
            m = best[groups["keep"] - 1] - best[groups["keep"]]
        choice = g[np.argsort(-g.max(axis=1), kind="stable")[:groups["keep"]]].reshape(-1)
    choice = np.sort(choice)[::-1]
    return min(m, choice[top - 1] - choice[top]) if top < len(choice) else m


def reference(cfg, w, tokens, taps=None):
    """(logits, per token the smallest margin of its routers)"""
    seen, choose = [], plain.choose

    def watched(z, correction, top, groups):
        seen.append(margin(z, correction, top, groups))
        return choose(z, correction, top, groups)
    plain.choose = watched
    try:
        logits = plain.forward(cfg, w, tokens, taps)
    finally:
        plain.choose = choose
    return logits, np.min(np.array(seen).reshape(-1, len(tokens)), axis=0) if seen else np.full(len(tokens), np.inf)


def agrees(got, want, dtype, margins):
    keep = np.asarray(margins) > (CLOSE if dtype == "bfloat16" else 0.0)
    assert keep.mean() > 0.5 or len(keep) < 10
    if not keep.any():
        return True
    d = (np.asarray(got, np.float64) - want)[keep]
    over = np.sqrt(np.mean(d * d, axis=-1)) / np.std(want) > LIMIT[dtype]
    return np.isfinite(got).all() and over.sum() <= (max(1, SHARE[dtype] * keep.sum()) if dtype == "bfloat16" else 0)


def setup(tmp_path_factory, name):
    """(cfg, weights, folder, tokens, logits of every position, residual streams, margins) of a configuration"""
    if name not in _cache:
        cfg = tm.configs()[name]
        w = tm.weights(cfg, 3)
        folder = str(tmp_path_factory.mktemp("tudasun_" + name))
        km.write(folder, cfg, w)
        tokens = np.random.default_rng(5).integers(0, cfg["vocab"], LENGTH).tolist()
        taps = []
        logits, margins = reference(cfg, w, tokens, taps)
        _cache[name] = (cfg, w, folder, tokens, logits, np.stack(taps), margins)
    return _cache[name]


@pytest.fixture(params=[(n, d) for n in NAMES for d in ("bfloat16", "float32")], ids=lambda p: "-".join(p))
def case(request, awq, torch_gpu, tmp_path_factory):
    name, dtype = request.param
    cfg, w, folder, tokens, logits, taps, margins = setup(tmp_path_factory, name)
    print("tudasun", name, dtype, flush=True)
    eng = awq.open_model(folder, dtype=dtype, max_positions=500)
    yield eng, cfg, tokens, logits, taps, dtype, margins
    eng.close()


def test_whole_prompt_and_every_layer(case):
    eng, cfg, tokens, logits, taps, dtype, margins = case
    assert eng.architecture == "Tudasun" and eng.vocab_size == cfg["vocab"] and eng.hidden_size == cfg["width"]
    assert agrees(eng.forward(tokens, range(len(tokens))), logits, dtype, margins)
    eng.set_layer_tap(True)
    eng.reset()
    eng.forward(tokens)
    got = eng.read_layer_tap().reshape(taps.shape)
    for i in range(len(taps)):
        assert agrees(got[i], taps[i], dtype, margins), "layer %d" % i
    # the same position by position (the one-token kernels)
    eng.reset()
    got = []
    for t in range(40):
        eng.forward(tokens[t:t + 1])
        got.append(eng.read_layer_tap().reshape(len(taps), cfg["width"]))
    got = np.stack(got, axis=1)
    for i in range(len(taps)):
        assert agrees(got[i], taps[i][:40], dtype, margins[:40]), "layer %d" % i


def test_decoding_agrees_with_the_prompt(case):
    eng, cfg, tokens, logits, taps, dtype, margins = case
    for cut in (0, 1, 63, 200):
        eng.reset()
        if cut:
            eng.forward(tokens[:cut])
        got = np.concatenate([eng.forward([t], [0]) for t in tokens[cut:]])
        assert agrees(got, logits[cut:], dtype, margins[cut:]), "from token %d" % cut


@pytest.mark.parametrize("sizes", [[2], [3, 2], [7, 1, 20], [64], [63, 65, 2], [17, 128], [150, 2]], ids=str)
def test_portions(case, sizes):
    eng, cfg, tokens, logits, taps, dtype, margins = case
    eng.reset()
    got, at, i = [], 0, 0
    while at < len(tokens):
        n = min(sizes[i % len(sizes)], len(tokens) - at)
        got.append(eng.forward(tokens[at:at + n], range(n)))
        at, i = at + n, i + 1
    assert agrees(np.concatenate(got), logits, dtype, margins)


def test_requests_one_after_the_other(case):
    """what an earlier request left in caches and states does not show in a later one"""
    eng, cfg, tokens, logits, taps, dtype, margins = case
    rng = np.random.default_rng(1)
    for n in (3, 150, 1, 70, 2, 331):
        eng.reset()
        eng.forward(rng.integers(0, cfg["vocab"], int(rng.integers(1, 500))).tolist())
        eng.reset()
        first = eng.forward(tokens[:n], range(n))
        eng.reset()
        again = eng.forward(tokens[:n], range(n))
        assert np.array_equal(first, again)
        assert agrees(first, logits[:n], dtype, margins[:n])


def test_graphs_and_eager_steps_give_the_same(case):
    eng, cfg, tokens, logits, taps, dtype, margins = case
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
    eng, cfg, tokens, logits, taps, dtype, margins = case
    w = _cache[[n for n in NAMES if tm.configs()[n] == cfg][0]][1]
    prompt = tokens[:37]
    for batched in (True, False):
        eng.set_prefill_mode(batched)
        out = eng.generateResponse(prompt, 130)
        assert len(out) == 130
        z, m = reference(cfg, w, prompt + out[:-1])
        z, m = z[len(prompt) - 1:], m[len(prompt) - 1:]
        short = z.max(axis=1) - z[np.arange(len(out)), out]
        decided = m > (CLOSE if dtype == "bfloat16" else 0.0)
        assert np.mean(short[decided] > 6 * LIMIT[dtype] * np.std(z)) <= SHARE[dtype]
        assert np.mean(short == 0) > (0.75 if dtype == "bfloat16" else 0.98)
    assert eng.generateResponse(prompt, 5) == out[:5]


def test_a_sequence_of_several_passes(awq, torch_gpu, tmp_path):
    """more positions than a pass of 2048 takes: states and cache rows go from pass to pass"""
    cfg = tm.model(32, 64, [tm.latent(2, 16, 8, 8, 40, mlp=tm.moe(4, 2, 16, 1)), tm.gla(1, 16, 8, 64.0), tm.hgrn2(2, 8, 8)], side=8)
    w = tm.weights(cfg, 3)
    w["l2.mix.lower"] = km.bf16(np.full(16, 0.99))   # remembers for hundreds of tokens
    km.write(str(tmp_path), cfg, w)
    tokens = np.random.default_rng(9).integers(0, cfg["vocab"], 2600).tolist()
    ref, margins = reference(cfg, w, tokens)
    for dtype in ("bfloat16", "float32"):
        eng = awq.open_model(str(tmp_path), dtype=dtype, max_positions=3000)
        got, at = [], 0
        for n in (2047, 100, 2, 1, 1, 1, 130, 2):
            got.append(eng.forward(tokens[at:at + n], range(n)))
            at += n
        while at < len(tokens):
            got.append(eng.forward(tokens[at:at + 1], [0]))
            at += 1
        assert agrees(np.concatenate(got), ref, dtype, margins)
        # one call, cut into passes by the engine
        eng.reset()
        assert agrees(eng.forward(tokens, range(len(tokens))), ref, dtype, margins)
        eng.close()


def test_float32_tensors_and_extra_keys(awq, torch_gpu, tmp_path):
    cfg = tm.model(48, 96, [tm.latent(2, 24, 4, 16, 20, mlp=tm.moe(3, 2, 10, 1, shared=6)), tm.gla(2, 12, 8, 3.0, tm.dense(20))], softcap=5.0)
    cfg["layers"][0]["mixer"]["unused"] = {"size": 3}
    w = tm.weights(cfg, 4)
    names = ("l0.mix.uk", "l0.mix.uv", "l0.mlp.e1.gate", "l1.norm1", "embed", "l1.mix.a2")
    for n in names:
        w[n] = (w[n] * np.float32(1.0001)).astype(np.float32)  # no longer bfloat16 values
    km.write(str(tmp_path), cfg, w, f32_names=names)
    tokens = list(range(30))
    eng = awq.open_model(str(tmp_path), dtype="float32", max_positions=64)
    assert agrees(eng.forward(tokens, range(30)), *reference(cfg, w, tokens)[:1], "float32", np.ones(30))
    with pytest.raises(awq.AwqError):
        eng.forward([0] * 35)             # does not fit max_positions
    eng.close()


def test_command_line_and_trace_runner(awq, torch_gpu, tmp_path):
    cfg = tm.model(64, 80, [tm.gla(2, 16, 24, 16.0, tm.moe(4, 2, 24, 2, (2, 1))), tm.latent(4, 16, 8, 16, 32, mlp=tm.dense(48)),
                            tm.hgrn2(2, 12, 16, tm.moe(3, 1, 20, shared=16))], softcap=4.0, side=5)
    w = tm.weights(cfg, 8)
    folder = str(tmp_path / "m")
    km.write(folder, cfg, w)
    pkg = os.path.join(ROOT, "cuda-kernel-qwen3-8b-awq_amd")
    run = subprocess.run([os.path.join(pkg, "qwen3_awq_infer"), folder, "--prompt", "3,1,4,1,5", "--new", "12", "--dtype", "float32"],
                         capture_output=True, text=True, timeout=100)
    assert run.returncode == 0, run.stderr
    ids = [int(t) for t in run.stdout.split(":")[1].split()]
    want, gap = plain.generate(cfg, w, [3, 1, 4, 1, 5], 12)
    assert gap > 1e-3 and ids == want
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
