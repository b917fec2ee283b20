"""Small Kugilix models for the tests: configurations, random weights, model folders."""
import json
import os
import struct

import numpy as np


def bf16(x):
    """rounded to bfloat16 (to nearest even), as float32"""
    u = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32).astype(np.uint64)
    u = (u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000
    return u.astype(np.uint32).view(np.float32)


def attention(heads, kv_heads, dim, vdim, window, scale=None, temp=(0.4, 16), ff=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else 2.0 / dim ** 0.5}
    if window:
        m["mask"] = {"size": window}
    if temp:
        m["q_temp"] = {"coef": temp[0], "every": temp[1]}
    return {"type": "attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def lightning(heads, dim, vdim, decay, ff=None):
    assert len(decay) == heads
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def model(width, vocab, layers, groups=2, taps=3, eps=1e-5, embed_scale=3.0, loop=None):
    cfg = {"architecture": "Kugilix", "vocab": vocab, "width": width, "canon": {"taps": taps},
           "embedding": {"scale": embed_scale}, "norm": {"eps": eps, "groups": groups}, "layers": layers}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def configs():
    """name -> configuration; together they take every branch and no two sizes of a layer are equal by habit"""
    return {
        # sizes that are multiples of nothing, more query heads than one workgroup takes, a loop in the middle
        "odd": model(90, 211, [lightning(3, 20, 12, [0.5, 0.9, 0.99], ff=70),
                               attention(6, 3, 20, 12, 17, ff=52),
                               attention(11, 1, 36, 44, 5, temp=None),
                               lightning(2, 9, 31, [0.8, 0.999])],
                     groups=5, taps=3, loop=(1, 3, 2)),
        # matrix-core sizes, several parts per window, loop over everything
        "even": model(256, 320, [attention(4, 2, 64, 128, 150, ff=384),
                                 lightning(2, 128, 64, [0.7, 0.995], ff=320)],
                      groups=4, taps=4, loop=(0, 2, 2)),
        # a window of one, no window, one head per group, a loop of one layer at the end, taps beyond the fast forms
        "edge": model(64, 128, [attention(2, 2, 128, 64, 1, ff=96), attention(2, 1, 64, 32, None, temp=(1.0, 3)),
                                lightning(1, 256, 40, [0.97], ff=64)],
                      groups=1, taps=10, loop=(2, 3, 3)),
        # no convolution reach, many heads of one key, long head rows
        "taps1": model(128, 200, [attention(12, 1, 16, 16, 66, ff=128), lightning(4, 40, 72, [0.25, 0.6, 0.9, 0.9995]),
                                  attention(1, 1, 200, 160, 40, ff=200)], groups=8, taps=1),
    }


def tensor_shapes(cfg):
    W, V, taps = cfg["width"], cfg["vocab"], cfg["canon"]["taps"]
    out = {"embed": (V, W), "final.norm": (W,), "head": (V, W)}
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], "l%d." % i
        H, D, VD = m["heads"], m["dim"], m["vdim"]
        G = m.get("kv_heads", H)
        out.update({p + "norm1": (W,), p + "canon1": (W, taps), p + "mix.q": (H * D, W), p + "mix.k": (G * D, W),
                    p + "mix.v": (G * VD, W), p + "mix.o": (W, H * VD)})
        if l["type"] == "lightning":
            out.update({p + "mix.g": (H * VD, W), p + "mix.norm": (H * VD,)})
        if l["mlp"]:
            ff = l["mlp"]["ff"]
            out.update({p + "norm2": (W,), p + "mlp.up": (ff, W), p + "mlp.down": (W, ff), p + "mlp.act": (2,)})
    return out


def weights(cfg, seed):
    """name -> float32 array of bfloat16 values"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        x = rng.standard_normal(shape)
        if name.endswith(("norm", "norm1", "norm2")):
            x = 1.0 + 0.3 * x
        elif name.endswith("canon1"):
            x = 0.4 * x
        elif name.endswith("act"):
            x = 0.7 * x
        elif name == "embed":
            x = 0.4 * x
        else:
            x = x / shape[1] ** 0.5
        out[name] = bf16(x)
    return out


def write(folder, cfg, w, f32_names=()):
    """config.json and model.safetensors; the tensors named in f32_names are stored as F32"""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, data = {}, []
    at = 0
    for name, x in w.items():
        wide = name in f32_names
        raw = x.astype("<f4").tobytes() if wide else (x.view(np.uint32) >> 16).astype("<u2").tobytes()
        header[name] = {"dtype": "F32" if wide else "BF16", "shape": list(x.shape), "data_offsets": [at, at + len(raw)]}
        at += len(raw)
        data.append(raw)
    head = json.dumps(header).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head + b"".join(data))


def rms_error(got, want):
    """root mean square difference over the spread of `want`, row by row; the largest row"""
    d = np.asarray(got, np.float64) - want
    return float(np.max(np.sqrt(np.mean(d * d, axis=-1))) / np.std(want))
