"""Small Tudasun models for the tests: configurations and random weights (folders are written by kugilix_model.write)."""
import numpy as np

from kugilix_model import bf16


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, identity=None, groups=None, shared=None):
    r = {"experts": experts, "top": top}
    if identity is not None:
        r["identity"] = identity
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    f = {"kind": "moe", "expert": {"ff": ff}, "router": r}
    if shared:
        f["shared"] = {"ff": shared}
    return f


def gla(heads, dim, vdim, tau, mlp=None):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "mlp": mlp}


def hgrn2(heads, dim, vdim, mlp=None):
    return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim}, "mlp": mlp}


def latent(heads, dim, rot, vdim, rank, base=10000.0, scale=None, kv_from=None, mlp=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "rot_dim": rot, "rot": {"base": base, "dims": rot},
         "scale": scale if scale is not None else 1.5 * (dim + rot) ** -0.5}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def model(width, vocab, layers, eps=1e-5, softcap=None, side=None):
    return {"architecture": "Tudasun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_softcap": softcap,
            "token_side": {"dim": side} if side else None, "layers": layers}


def configs():
    """name -> configuration; together they take every branch and no two sizes of a layer are equal by habit"""
    return {
        # sizes that are multiples of nothing; a layer without feed-forward; no identity outputs, no groups, no shared expert
        "odd": model(90, 211, [gla(3, 20, 12, 4.0, dense(70)), latent(3, 19, 6, 13, 37, 500.0, mlp=moe(5, 2, 21)),
                               hgrn2(2, 9, 31), latent(5, 11, 6, 7, 37, 500.0, kv_from=1, mlp=moe(7, 3, 10, identity=2, shared=17)),
                               gla(1, 33, 5, 1.0, moe(3, 2, 30, identity=3, groups=(3, 1)))], eps=1e-3, softcap=2.0, side=7),
        # sizes of the matrix-core forms, keys and values formed for long passes, two layers on one layer's latents
        "even": model(256, 320, [latent(4, 64, 32, 64, 128, mlp=dense(384)),
                                 latent(2, 96, 32, 128, 128, kv_from=0, mlp=moe(12, 3, 64, identity=4, groups=(4, 2), shared=128)),
                                 hgrn2(4, 64, 64, moe(6, 4, 72, identity=2, groups=(4, 3), shared=64)),
                                 gla(2, 128, 96, 8.0, moe(8, 2, 64, shared=40)),
                                 latent(8, 32, 32, 24, 128, kv_from=0)], softcap=3.0, side=64),
        # one head; a latent wider than a workgroup's threads; states of 200 rows; every output chosen; no cap, no token input
        "edge": model(64, 128, [hgrn2(1, 200, 40, moe(2, 4, 24, identity=2, shared=8)), latent(1, 40, 2, 48, 300, 7.0),
                                gla(1, 64, 72, 6.0, dense(33)), latent(2, 72, 64, 8, 60, 50000.0, mlp=moe(4, 1, 16, groups=(2, 1)))],
                      eps=1e-6),
    }


def tensor_shapes(cfg, low=5):
    W, V, L, S = cfg["width"], cfg["vocab"], len(cfg["layers"]), (cfg["token_side"] or {}).get("dim")
    out = {"embed": (V, W), "final.norm": (W,), "head": (V, W)}
    if S:
        out["side.embed"] = (V, L * S)
    for i, l in enumerate(cfg["layers"]):
        m, f, p = l["mixer"], l["mlp"], "l%d." % i
        keys, mixed = m["heads"] * m["dim"], m["heads"] * m["vdim"]
        out.update({p + "norm1": (W,), p + "norm1b": (W,), p + "rg1": (W, W), p + "rg1.b": (W,), p + "mix.o": (W, mixed)})
        if l["type"] == "latent_attention":
            out.update({p + "mix.q": (keys + m["heads"] * m["rot_dim"], W), p + "mix.uk": (keys, m["kv_rank"]),
                        p + "mix.uv": (mixed, m["kv_rank"]), p + "mix.sink": (m["heads"],)})
            if "kv_from" not in m:
                out.update({p + "mix.dkv": (m["kv_rank"] + m["rot_dim"], W), p + "mix.dkv.norm": (m["kv_rank"],)})
        else:
            out.update({p + "mix.q": (keys, W), p + "mix.v": (mixed, W), p + "mix.norm": (m["vdim"],)})
            if l["type"] == "gla":
                out.update({p + "mix.k": (keys, W), p + "mix.g": (mixed, W), p + "mix.a1": (low, W), p + "mix.a2": (keys, low),
                            p + "mix.a2.b": (keys,)})
            else:
                out.update({p + "mix.f": (keys, W), p + "mix.f.b": (keys,), p + "mix.lower": (keys,)})
        if f:
            out.update({p + "norm2": (W,), p + "norm2b": (W,), p + "rg2": (W, W), p + "rg2.b": (W,)})
            if f["kind"] == "dense":
                out.update({p + "mlp.up": (f["ff"], W), p + "mlp.down": (W, f["ff"]), p + "mlp.act": (4,)})
            else:
                n = f["router"]["experts"] + f["router"].get("identity", 0)
                out.update({p + "mlp.router": (n, W), p + "mlp.correction": (n,)})
                sizes = {"e%d" % e: f["expert"]["ff"] for e in range(f["router"]["experts"])}
                if "shared" in f:
                    sizes["shared"] = f["shared"]["ff"]
                    out[p + "mlp.shared.sg"] = (1, W)
                for e, ff in sizes.items():
                    out.update({p + "mlp.%s.gate" % e: (ff, W), p + "mlp.%s.up" % e: (ff, W), p + "mlp.%s.down" % e: (W, ff)})
        if S:
            out.update({p + "side.gate": (S, W), p + "side.proj": (W, S), p + "side.norm": (W,)})
    return out


def weights(cfg, seed):
    """name -> float32 array of bfloat16 values"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        x = rng.standard_normal(shape)
        if name.endswith(("mix.norm", "dkv.norm", "side.norm")):
            x = 1.0 + 0.3 * x
        elif name.endswith(("norm", "norm1", "norm2", "norm1b", "norm2b")):
            x = 0.3 * x                                  # around zero
        elif name.endswith("lower"):
            x = np.maximum(0.0, rng.random(shape) - 0.2)
        elif name.endswith("correction"):
            x = 1.0 * x
        elif name.endswith("mlp.act"):
            x = 0.7 * x + 0.3
        elif name.endswith("router"):
            x = 3.0 * x / shape[1] ** 0.5                # far from close calls, mostly
        elif name.endswith("a2.b"):
            x = 2.0 * x + 2.0
        elif name.endswith("sink"):
            x = 1.5 * x
        elif len(shape) == 2 and name != "embed":
            x = x / shape[1] ** 0.5
        out[name] = bf16(x)
    return out
