#!/usr/bin/env python3
"""Prompt and decode throughput of the Tudasun design at the sizes of real models' layers, beside the Kugilix model (the
framework's closest one) at equal width, heads, vocabulary and number of layers.

Random weights, written once as a model folder and opened the way a user's folder is.  Four layers take every mechanism:
gated linear attention with a dense feed-forward, latent attention, latent attention on the latents of the layer ahead,
and HGRN2, the last three with routed experts.  A token meets up to 11.25 width^2
feed-forward weights in an expert layer (four experts and the shared one, each three matrices of 3/4 width), 6 in the dense one.

Run on the GPU box: python bench.py --mode tudasun [--tudasun-sizes 2048,4096] [--tudasun-only]
"""
import importlib
import os
import sys
import tempfile

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
sys.path.insert(0, ROOT)

from . import bench_kugilix as closest

HEAD, VOCAB, RANK, ROT, SIDE, LOW = 128, 32768, 512, 64, 256, 16
EXPERTS, IDENTITY, TOP = 14, 2, 4


def config(width, repeat=1):
    heads = width // HEAD
    linear = {"heads": heads, "dim": HEAD, "vdim": HEAD}
    latent = {"heads": heads, "dim": HEAD, "vdim": HEAD, "kv_rank": RANK, "rot_dim": ROT, "scale": (HEAD + ROT) ** -0.5,
              "rot": {"base": 10000.0, "dims": ROT}}
    moe = {"kind": "moe", "expert": {"ff": 3 * width // 4}, "shared": {"ff": 3 * width // 4},
           "router": {"experts": EXPERTS, "identity": IDENTITY, "top": TOP, "groups": {"count": 4, "keep": 2}}}
    layers = []
    for _ in range(repeat):
        n = len(layers)
        layers += [{"type": "gla", "mixer": dict(linear, tau=16.0), "mlp": {"kind": "dense", "ff": 3 * width}},
                   {"type": "latent_attention", "mixer": latent, "mlp": moe},
                   {"type": "latent_attention", "mixer": dict(latent, kv_from=n + 1), "mlp": moe},
                   {"type": "hgrn2", "mixer": linear, "mlp": moe}]
    return {"architecture": "Tudasun", "vocab": VOCAB, "width": width, "norm": {"eps": 1e-6}, "logit_softcap": 30.0,
            "token_side": {"dim": SIDE}, "layers": layers}


def shapes(cfg):
    W, V, L = cfg["width"], cfg["vocab"], len(cfg["layers"])
    out = {"embed": [V, W], "final.norm": [W], "head": [V, W], "side.embed": [V, L * SIDE]}
    for i, l in enumerate(cfg["layers"]):
        m, f, p = l["mixer"], l["mlp"], "l%d." % i
        keys, mixed = m["heads"] * m["dim"], m["heads"] * m["vdim"]
        for n in ("norm1", "norm1b", "norm2", "norm2b", "rg1.b", "rg2.b", "side.norm"):
            out[p + n] = [W]
        out.update({p + "rg1": [W, W], p + "rg2": [W, W], p + "side.gate": [SIDE, W], p + "side.proj": [W, SIDE],
                    p + "mix.o": [W, mixed]})
        if l["type"] == "latent_attention":
            out.update({p + "mix.q": [m["heads"] * (m["dim"] + ROT), W], p + "mix.uk": [keys, RANK], p + "mix.uv": [mixed, RANK],
                        p + "mix.sink": [m["heads"]]})
            if "kv_from" not in m:
                out.update({p + "mix.dkv": [RANK + ROT, W], p + "mix.dkv.norm": [RANK]})
        else:
            out.update({p + "mix.q": [keys, W], p + "mix.v": [mixed, W], p + "mix.norm": [m["vdim"]]})
            if l["type"] == "gla":
                out.update({p + "mix.k": [keys, W], p + "mix.g": [mixed, W], p + "mix.a1": [LOW, W], p + "mix.a2": [keys, LOW],
                            p + "mix.a2.b": [keys]})
            else:
                out.update({p + "mix.f": [keys, W], p + "mix.f.b": [keys], p + "mix.lower": [keys]})
        if f["kind"] == "dense":
            out.update({p + "mlp.up": [f["ff"], W], p + "mlp.down": [W, f["ff"]], p + "mlp.act": [4]})
        else:
            n = f["router"]["experts"] + f["router"]["identity"]
            out.update({p + "mlp.router": [n, W], p + "mlp.correction": [n], p + "mlp.shared.sg": [1, W]})
            for e in ["e%d" % e for e in range(f["router"]["experts"])] + ["shared"]:
                ff = f["expert"]["ff"] if e != "shared" else f["shared"]["ff"]
                out.update({p + "mlp.%s.gate" % e: [ff, W], p + "mlp.%s.up" % e: [ff, W], p + "mlp.%s.down" % e: [W, ff]})
    return out


def active_params(cfg):
    """matrix weights that one token meets: of the experts, those of `top` outputs (identity outputs among them)"""
    n = 0
    for name, s in shapes(cfg).items():
        if len(s) != 2 or "embed" in name:
            continue
        k = s[0] * s[1]
        if ".mlp.e" in name:
            r = cfg["layers"][int(name[1:name.index(".")])]["mlp"]["router"]
            k = k * r["top"] / (r["experts"] + r["identity"])
        n += k
    return n


def measure(widths, only=False, prompts=(128, 1024), steps=128):
    awq = importlib.import_module("cuda-kernel-qwen3-8b-awq_amd")
    res = {}
    positions = max(prompts) + 8 + 2 * steps
    for width in widths:
        models = [("tudasun", config(width), shapes, active_params)]
        if not only:
            models.append(("kugilix", closest.config(width, n_layers=4), closest.shapes, closest.matrix_params))
        for name, cfg, shapes_of, params_of in models:
            print("model", name, width, file=sys.stderr, flush=True)
            with tempfile.TemporaryDirectory() as d:
                closest.write_model(d, cfg, shapes_of=shapes_of)
                eng = awq.open_model(d, max_positions=positions)
            r = closest.run_engine(eng, VOCAB, prompts, steps)
            eng.close()
            params = params_of(cfg)
            r["decode_hbm_fraction"] = round(2 * params / (r["decode_us"] * 1e-6) / closest.HBM, 3)
            body = params - VOCAB * width   # prompt positions other than the sampled one do not meet the head
            for P in prompts:
                r["prefill_%d_mfma_fraction" % P] = round(2 * body * P / (r["prefill_%d_ms" % P] * 1e-3) / closest.MFMA, 3)
            r["active_matrix_params"] = int(params)
            res["%s_%d" % (name, width)] = r
    return {"layers": 4, "vocab": VOCAB, "head_dim": HEAD, "kv_rank": RANK, "experts": EXPERTS, "top": TOP, "results": res}
