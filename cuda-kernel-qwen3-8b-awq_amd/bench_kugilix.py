#!/usr/bin/env python3
"""Prompt and decode throughput of the Kugilix design at the sizes of real models' layers, beside the int4 model
(the framework's closest one) at equal width, feed-forward, heads, vocabulary and number of layers.

Random weights, written once as a model folder (config.json + model.safetensors) and opened the way a user's
folder is.  Half the layers are attention over a window, half linear attention; no layer is repeated, so that both
models do the same number of products.  The bytes and operations of a step come from the shapes; peaks: 8 TB/s,
2.5 PFLOP/s dense at 16 bits.

Run on the GPU box: python bench.py --mode kugilix [--kugilix-sizes 2048,4096] [--kugilix-only]
"""
import importlib
import json
import os
import struct
import sys
import tempfile
import time

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
sys.path.insert(0, ROOT)

HBM = 8e12
MFMA = 2.5e15
LAYERS, VOCAB, WINDOW, HEAD = 8, 32768, 1024, 128


def config(width, kv_heads=None, n_layers=LAYERS, window=WINDOW, vocab=VOCAB):
    heads = width // HEAD
    att = {"type": "attention",
           "mixer": {"heads": heads, "kv_heads": kv_heads or heads, "dim": HEAD, "vdim": HEAD, "scale": HEAD ** -0.5,
                     "mask": {"size": window}, "q_temp": {"coef": 0.1, "every": 512}},
           "mlp": {"kind": "dense", "ff": 3 * width}}
    lin = {"type": "lightning",
           "mixer": {"heads": heads, "dim": HEAD, "vdim": HEAD,
                     "decay": [1.0 - 2.0 ** (-1.0 - 7.0 * h / heads) for h in range(heads)]},
           "mlp": {"kind": "dense", "ff": 3 * width}}
    return {"architecture": "Kugilix", "vocab": vocab, "width": width, "canon": {"taps": 4},
            "embedding": {"scale": 1.0}, "norm": {"eps": 1e-6, "groups": 8},
            "layers": [att if i % 2 == 0 else lin for i in range(n_layers)],
            "loop": {"start": 0, "stop": 0, "times": 1}}


def shapes(cfg):
    W, V, taps = cfg["width"], cfg["vocab"], cfg["canon"]["taps"]
    out = {"embed": [V, W], "final.norm": [W], "head": [V, W]}
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], "l%d." % i
        g = m.get("kv_heads", m["heads"])
        out[p + "norm1"] = [W]
        out[p + "canon1"] = [W, taps]
        out[p + "mix.q"] = [m["heads"] * m["dim"], W]
        out[p + "mix.k"] = [g * m["dim"], W]
        out[p + "mix.v"] = [g * m["vdim"], W]
        out[p + "mix.o"] = [W, m["heads"] * m["vdim"]]
        if l["type"] == "lightning":
            out[p + "mix.g"] = [m["heads"] * m["vdim"], W]
            out[p + "mix.norm"] = [m["heads"] * m["vdim"]]
        if l.get("mlp"):
            ff = l["mlp"]["ff"]
            out[p + "norm2"] = [W]
            out[p + "mlp.up"] = [ff, W]
            out[p + "mlp.down"] = [W, ff]
            out[p + "mlp.act"] = [2]
    return out


def write_model(folder, cfg, seed=0, shapes_of=shapes):
    """config.json and model.safetensors with random weights (one block of normal numbers, reused at offsets)"""
    import numpy as np
    rng = np.random.default_rng(seed)
    pool = rng.standard_normal(1 << 24, dtype=np.float32)
    sh = shapes_of(cfg)
    header, at = {}, 0
    for name, s in sh.items():
        n = 2 * int(np.prod(s))
        header[name] = {"dtype": "BF16", "shape": s, "data_offsets": [at, at + n]}
        at += n
    head = json.dumps(header).encode()
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head)
        for name, s in sh.items():
            n = int(np.prod(s))
            scale = 0.02 if name == "embed" else (s[1] ** -0.5 if len(s) == 2 else 0.1)
            shift = 1.0 if name.endswith(("norm", "norm1", "norm2")) else 0.5 if name.endswith("lower") else 0.0
            while n > 0:
                k = min(n, pool.size // 2)
                o = int(rng.integers(0, pool.size - k))
                bits = (pool[o:o + k] * np.float32(scale) + np.float32(shift)).view(np.uint32)
                f.write((bits >> 16).astype(np.uint16).tobytes())
                n -= k


def matrix_params(cfg):
    return sum(s[0] * s[1] for name, s in shapes(cfg).items() if len(s) == 2 and name != "embed" and "canon" not in name)


def timed(fn, reps=3):
    best = 1e9
    for _ in range(reps):
        t = time.perf_counter()
        fn()
        best = min(best, time.perf_counter() - t)
    return best


def run_engine(eng, vocab, prompts, steps):
    out = {}
    for P in prompts:
        prompt = [(7 * i + 3) % vocab for i in range(P)]

        def once():
            eng.reset()
            eng.prefill(prompt, batched=True)   # returns after the device finished
        once()
        out["prefill_%d_ms" % P] = round(1e3 * timed(once), 3)
    eng.decode(8)
    out["decode_us"] = round(1e6 * timed(lambda: eng.decode(steps), 2) / steps, 1)
    out["decode_from_position"] = prompts[-1]
    return out


def measure(widths, only=False, prompts=(128, 1024), steps=128):
    awq = importlib.import_module("cuda-kernel-qwen3-8b-awq_amd")
    lib = awq.load_library()
    from bench import _synthetic_engine
    res = {}
    positions = max(prompts) + 8 + 2 * steps
    for width in widths:
        cfg = config(width)
        with tempfile.TemporaryDirectory() as d:
            write_model(d, cfg)
            eng = awq.open_model(d, max_positions=positions)
        r = run_engine(eng, VOCAB, prompts, steps)
        eng.close()
        params = matrix_params(cfg)
        r["decode_hbm_fraction"] = round(2 * params / (r["decode_us"] * 1e-6) / HBM, 3)
        body = params - cfg["vocab"] * width   # prompt positions other than the sampled one do not meet the head
        for P in prompts:
            r["prefill_%d_mfma_fraction" % P] = round(2 * body * P / (r["prefill_%d_ms" % P] * 1e-3) / MFMA, 3)
        res["kugilix_%d" % width] = r
        if only:
            continue
        c = awq.make_config(n_layers=LAYERS, hidden=width, inter=3 * width, vocab=VOCAB, max_pos=positions)
        eng = _synthetic_engine(awq, lib, c, 1, awq.SYNTH_BALANCED)
        r = run_engine(eng, VOCAB, prompts, steps)
        eng.close()
        body = LAYERS * (4 * width * width + 2 * 3 * width * width)
        params = body + VOCAB * width
        r["decode_hbm_fraction"] = round(0.5 * params / (r["decode_us"] * 1e-6) / HBM, 3)
        for P in prompts:
            r["prefill_%d_mfma_fraction" % P] = round(2 * body * P / (r["prefill_%d_ms" % P] * 1e-3) / MFMA, 3)
        res["int4_%d" % width] = r
    return {"layers": LAYERS, "vocab": VOCAB, "window": WINDOW, "head_dim": HEAD, "results": res}
