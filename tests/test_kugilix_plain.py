"""The plain statement itself (kugilix_plain.py), and what the engine checks of a model folder before it touches a
GPU."""
import ctypes
import json
import os
import subprocess

import numpy as np
import pytest

import kugilix_model as km
import kugilix_plain as plain


def test_linear_attention_is_the_decayed_sum():
    rng = np.random.default_rng(0)
    q, k, v = rng.standard_normal((3, 9, 2, 4))
    decay = [0.5, 0.9]
    o, S = plain.linear_attention(q, k, v, decay)
    for h in range(2):
        for t in range(9):
            want = sum(decay[h] ** (t - s) * (k[s, h] @ q[t, h]) * v[s, h] for s in range(t + 1))
            assert np.allclose(o[t, h], want)
    a, mid = plain.linear_attention(q[:4], k[:4], v[:4], decay)
    b, end = plain.linear_attention(q[4:], k[4:], v[4:], decay, mid)
    assert np.allclose(np.concatenate([a, b]), o) and np.allclose(end, S)


def test_window_attention_by_hand():
    rng = np.random.default_rng(1)
    q, k, v = rng.standard_normal((7, 2, 3)), rng.standard_normal((7, 1, 3)), rng.standard_normal((7, 1, 2))
    o = plain.window_attention(q, k, v, 3, 0.7, (0.2, 2))
    i, h = 5, 1
    z = 1 + 0.2 * np.log(np.floor(6 / 2) + 1)
    s = np.array([k[j, 0] @ q[i, h] * z * 0.7 - 2.0 ** -8 * (i - j) for j in (3, 4, 5)])
    p = np.exp(s) / np.exp(s).sum()
    assert np.allclose(o[i, h], p @ v[3:6, 0])
    assert np.allclose(o[0], v[0, 0])


def test_convolution_and_norm():
    h = np.arange(12.0).reshape(6, 2)
    w = np.array([[1.0, 10.0, 100.0], [0.0, 0.0, 2.0]])
    y = plain.causal_conv(h, w)
    assert y[0, 0] == 0 and y[3, 0] == h[3, 0] + h[1, 0] + 10 * h[2, 0] + 100 * h[3, 0]
    assert np.allclose(y[:, 1], 3 * h[:, 1])
    assert np.allclose(plain.causal_conv(h[4:], w, h[2:4]), y[4:])
    x = np.array([[3.0, 4.0, 0.0, 2.0]])
    got = plain.grouped_norm(x, np.ones(4), 2, 0.5)
    assert np.allclose(got, [[3 / np.sqrt(13), 4 / np.sqrt(13), 0, 2 / np.sqrt(2.5)]])


def test_activation_and_positions():
    assert np.isclose(plain.xielu(np.array(2.0), 0.3, 9.0), np.log1p(np.exp(0.3)) * 4 + 1)
    assert np.isclose(plain.xielu(np.array(-2.0), 9.0, 0.3), (0.5 + np.log1p(np.exp(0.3))) * (np.exp(-2) - 1 + 2) - 1)
    s = plain.sinusoid(5, 6)
    assert np.isclose(s[2], np.sin(5 * 10000 ** (-2 / 6))) and np.isclose(s[3], np.cos(5 * 10000 ** (-2 / 6)))


def test_loop_order():
    cfg = {"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 3}}
    assert plain.layer_runs(cfg) == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False)]


@pytest.mark.parametrize("name", sorted(km.configs()))
def test_the_test_models_tell_mistakes_apart(name):
    """A window that is one off, a dropped state, a temperature left out: each moves some logits by far more than the
    bfloat16 limit of the device tests (planted here, in the plain statement)."""
    cfg = km.configs()[name]
    w = km.weights(cfg, 11 + sorted(km.configs()).index(name))
    tokens = np.random.default_rng(5).integers(0, cfg["vocab"], 160).tolist()
    ref = plain.forward(cfg, w, tokens)

    def moved(change):
        other = json.loads(json.dumps(cfg))
        change(other)
        return km.rms_error(plain.forward(other, w, tokens), ref)

    def window(by):
        def f(c):
            for l in c["layers"]:
                if l["mixer"].get("mask"):
                    l["mixer"]["mask"]["size"] = max(1, l["mixer"]["mask"]["size"] + by)
        return f

    def decay(c):
        for l in c["layers"]:
            if "decay" in l["mixer"]:
                l["mixer"]["decay"] = [d * 0.5 for d in l["mixer"]["decay"]]

    def temperature(c):
        for l in c["layers"]:
            l["mixer"].pop("q_temp", None)

    assert moved(decay) > 0.1
    assert moved(temperature) > 0.03
    if name != "taps1":  # windows as wide as these hide a key at the edge; the single-mechanism tests show it
        if name != "even":
            assert moved(window(1)) > 0.03
    if cfg.get("loop"):
        assert moved(lambda c: c["loop"].update(times=c["loop"]["times"] + 1)) > 0.1


def open_rc(awq, lib, folder):
    h = ctypes.c_void_p()
    rc = lib.awq_open(os.fsencode(str(folder)), None, ctypes.byref(h))
    assert rc != 0 and not h.value
    return rc, lib.awq_last_error().decode()


def test_folders_are_checked_before_the_gpu(awq, lib, tmp_path):
    good = km.model(24, 30, [km.attention(2, 1, 8, 6, 5, ff=16), km.lightning(2, 4, 6, [0.5, 0.9])], groups=3, loop=(0, 1, 2))
    w = km.weights(good, 0)

    def bad(change, *words, drop=None, shapes=None):
        cfg, ww = json.loads(json.dumps(good)), dict(w)
        change(cfg)
        if drop:
            ww.pop(drop)
        if shapes:
            ww[shapes] = ww[shapes][:-1]
        km.write(str(tmp_path), cfg, ww)
        rc, message = open_rc(awq, lib, tmp_path)
        assert all(x in message for x in words), message
        return rc

    assert bad(lambda c: c.update(architecture="Nothing"), "no model class", "Nothing") == 1
    assert bad(lambda c: c.pop("architecture"), "no architecture") == 1
    assert bad(lambda c: c.pop("width"), "width") == 1
    assert bad(lambda c: c.update(width=24.5), "width") == 1
    assert bad(lambda c: c["norm"].update(groups=7), "norm.groups") == 1
    assert bad(lambda c: c["canon"].update(taps=0), "taps") == 1
    assert bad(lambda c: c["layers"].clear(), "layers") == 1
    assert bad(lambda c: c["layers"][0].update(type="other"), "layers[0].type", "other") == 1
    assert bad(lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "kv_heads") == 1
    assert bad(lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "mask.size") == 1
    assert bad(lambda c: c["layers"][1]["mixer"]["decay"].pop(), "decay") == 1
    assert bad(lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "mlp.kind") == 1
    assert bad(lambda c: c["loop"].update(stop=3), "loop.stop") == 1
    assert bad(lambda c: None, "l1.mix.g", drop="l1.mix.g") == 2
    assert bad(lambda c: None, "final.norm", "shape", shapes="final.norm") == 2
    km.write(str(tmp_path), good, w)
    path = tmp_path / "model.safetensors"
    raw = path.read_bytes()
    for cut in (raw[:5], raw[:100], raw[:-2], b"\xff" * 8 + raw[8:], raw[:8] + b"!" + raw[9:]):
        path.write_bytes(cut)
        assert open_rc(awq, lib, tmp_path)[0] == 2
    (tmp_path / "config.json").write_text("{\"architecture\": \"Kugilix\",}")
    assert open_rc(awq, lib, tmp_path)[0] == 1
    (tmp_path / "config.json").unlink()   # without one it is a raw weight directory, and an empty one
    assert "could not open" in open_rc(awq, lib, tmp_path)[1]


def test_trace_runner_refuses_what_it_cannot_do(tmp_path):
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    runner = os.path.join(root, "bin", "trace_run")

    def rc(*args):
        run = subprocess.run([runner, *args], input="", capture_output=True, text=True, timeout=60)
        assert run.stderr
        return run.returncode

    assert rc("--model", str(tmp_path)) == 1                                         # no --out
    assert rc("--model", str(tmp_path), "--out", str(tmp_path), "--dtype", "int8") == 1
    assert rc("--model", str(tmp_path), "--out", str(tmp_path), "--speed", "1") == 1
    assert rc("--model", str(tmp_path / "none"), "--out", str(tmp_path)) == 1
