"""The plain statement itself (tudasun_plain.py), and what the engine checks of a Tudasun folder before it touches a GPU."""
import json

import numpy as np
import pytest

import kugilix_model as km
import tudasun_model as tm
import tudasun_plain as plain
from test_kugilix_plain import open_rc


def test_gated_state_is_the_decayed_sum():
    rng = np.random.default_rng(0)
    q, k, v = rng.standard_normal((7, 2, 3)), rng.standard_normal((7, 2, 3)), rng.standard_normal((7, 2, 4))
    a = rng.random((7, 2, 3))
    o, S = plain.gated_state(q, k, v, a)
    for h in range(2):
        for t in range(7):
            want = sum((q[t, h] * np.prod(a[s + 1:t + 1, h], axis=0) * k[s, h]).sum() * v[s, h] for s in range(t + 1))
            assert np.allclose(o[t, h], want)
    _, mid = plain.gated_state(q[:3], k[:3], v[:3], a[:3])
    b, end = plain.gated_state(q[3:], k[3:], v[3:], a[3:], mid)
    assert np.allclose(b, o[3:]) and np.allclose(end, S)


def test_decays():
    assert np.isclose(plain.gla_decay(np.array(0.7), 16.0), (1 / (1 + np.exp(-0.7))) ** 0.0625)
    assert np.isclose(plain.hgrn2_forget(np.array(-0.4), 0.25), 0.25 + 0.75 / (1 + np.exp(0.4)))


def test_rotation_and_sink():
    x = np.array([[1.0, 2.0, 3.0, 4.0]])
    y = plain.rotate(x, 5, 100.0)[0]
    a, b = 5.0, 5.0 * 100.0 ** -0.5
    assert np.allclose(y, [np.cos(a) - 2 * np.sin(a), 2 * np.cos(a) + np.sin(a), 3 * np.cos(b) - 4 * np.sin(b), 4 * np.cos(b) + 3 * np.sin(b)])
    w = plain.softmax_with_sink(np.array([0.0, 1.0]), 2.0)
    assert np.allclose(w, np.exp([0, 1]) / (np.exp(0) + np.exp(1) + np.exp(2)))


def test_latent_attention_by_hand():
    rng = np.random.default_rng(1)
    qn, qr = rng.standard_normal((2, 1, 3)), rng.standard_normal((2, 1, 2))
    c, kr = rng.standard_normal((4, 5)), rng.standard_normal((4, 2))
    uk, uv = rng.standard_normal((1, 3, 5)), rng.standard_normal((1, 2, 5))
    o = plain.latent_attention(qn, qr, c, kr, uk, uv, 0.4, [0.3], 2)
    s = np.array([(uk[0] @ c[j]) @ qn[0, 0] + kr[j] @ qr[0, 0] for j in range(3)]) * 0.4
    assert np.allclose(o[0, 0], np.exp(s) @ (c[:3] @ uv[0].T) / (np.exp(s).sum() + np.exp(0.3)))


def test_router_choice():
    z = np.log(np.array([0.10, 0.30, 0.05, 0.25, 0.20, 0.10]))
    s = np.exp(z)
    assert plain.choose(z, None, 2, None) == [(1, pytest.approx(0.3 / 0.55)), (3, pytest.approx(0.25 / 0.55))]
    # the correction decides the choice, not the weights; negative choice scores still beat the outputs that are left out
    got = plain.choose(z, np.array([-1, -1, -0.5, -1, -1, -1.0]), 2, {"count": 3, "keep": 1})
    assert [i for i, _ in got] == [2, 3] and np.allclose([w for _, w in got], s[[2, 3]] / s[[2, 3]].sum())


def test_polynorm_and_gelu():
    z = np.array([[1.0, -2.0, 3.0]])
    n = lambda v: v / np.sqrt((v ** 2).mean() + 0.5)
    assert np.allclose(plain.polynorm(z, (2, 3, 4, 5), 0.5), 2 * n(z) + 3 * n(z ** 2) + 4 * n(z ** 3) + 5)
    assert np.isclose(plain.gelu_tanh(np.array(1.3)), 0.65 * (1 + np.tanh(np.sqrt(2 / np.pi) * (1.3 + 0.044715 * 2.197))))


@pytest.mark.parametrize("name", sorted(tm.configs()))
def test_the_test_models_tell_mistakes_apart(name, monkeypatch):
    """each mistake, planted here in the plain statement or its inputs, moves some logits by far more than the limit of the
    device tests"""
    cfg = tm.configs()[name]
    w = tm.weights(cfg, 3)
    tokens = np.random.default_rng(5).integers(0, cfg["vocab"], 60).tolist()
    ref = plain.forward(cfg, w, tokens)

    def moved(change_cfg=None, change_w=None, patch=None):
        other, ww = json.loads(json.dumps(cfg)), dict(w)
        if change_cfg:
            change_cfg(other)
        if change_w:
            change_w(ww)
        with monkeypatch.context() as m:
            if patch:
                m.setattr(plain, *patch)
            return km.rms_error(plain.forward(other, ww, tokens), ref)

    def without(*ends):
        def f(ww):
            for k in ww:
                if k.endswith(ends):
                    ww[k] = np.zeros_like(ww[k])
        return f

    def no_sinks(ww):
        for k in [k for k in ww if k.endswith("sink")]:
            del ww[k]

    def mixers(kind, f):
        def g(c):
            for l in c["layers"]:
                if l["type"] == kind:
                    f(l)
        return g

    def forget(q, k, v, decay, state=None):
        return gated(q, k, v, 0.0 * decay, state)

    gated = plain.gated_state
    assert moved(change_w=no_sinks) > 0.1
    assert moved(patch=("gated_state", forget)) > 0.1
    assert moved(patch=("norm", lambda x, g, eps: plain.rms(x, eps) * g)) > 0.1
    assert moved(patch=("rotate", lambda x, p, base: x)) > 0.1
    assert moved(mixers("gla", lambda l: l["mixer"].update(tau=0.25 * l["mixer"]["tau"]))) > 0.1
    assert moved(change_w=without("lower")) > 0.1
    assert moved(change_w=without("f.b", "a2.b")) > 0.1
    assert moved(change_w=without("correction")) > 0.1
    assert moved(change_w=without("rg1.b", "rg2.b")) > 0.1
    assert moved(change_w=without("mlp.act")) > 0.1
    if name != "edge":
        assert moved(lambda c: c.update(logit_softcap=None)) > 0.01
        assert moved(lambda c: c.update(token_side=None)) > 0.1
        assert moved(change_w=lambda ww: ww.update({"side.embed": np.roll(ww["side.embed"], cfg["token_side"]["dim"], axis=1)})) > 0.1

    def no_groups(c):
        for l in c["layers"]:
            if l["mlp"] and l["mlp"]["kind"] == "moe":
                l["mlp"]["router"].pop("groups", None)

    def own_scores(z, correction, top, groups):  # weights from the corrected scores
        ids = [i for i, _ in choose(z, correction, top, groups)]
        s = np.exp(z - z.max())
        s = s / s.sum() + correction
        return [(i, s[i] / (s[ids].sum() + 1e-20)) for i in ids]

    choose = plain.choose
    if name != "edge":  # (there the best output lies in the best group)
        assert moved(no_groups) > 0.1
    assert moved(patch=("choose", own_scores)) > 0.1
    if any("shared" in (l["mlp"] or {}) for l in cfg["layers"]):
        assert moved(change_w=without("shared.sg")) > 0.1


def test_folders_are_checked_before_the_gpu(awq, lib, tmp_path):
    good = tm.model(24, 30, [tm.gla(2, 4, 6, 2.0, tm.dense(9)), tm.latent(2, 4, 2, 3, 10, mlp=tm.moe(4, 2, 5, 2, (3, 1), 7)),
                             tm.latent(1, 4, 2, 3, 10, kv_from=1), tm.hgrn2(2, 3, 5)], softcap=5.0, side=3)
    w = tm.weights(good, 0)

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

    layer = lambda c, i: c["layers"][i]["mixer"]
    router = lambda c: c["layers"][1]["mlp"]["router"]
    assert bad(lambda c: c.pop("width"), "width") == 1
    assert bad(lambda c: c.pop("norm"), "norm") == 1
    assert bad(lambda c: c.update(logit_softcap=-1.0), "logit_softcap") == 1
    assert bad(lambda c: c["token_side"].update(dim=0), "token_side.dim") == 1
    assert bad(lambda c: c["layers"].clear(), "layers") == 1
    assert bad(lambda c: c["layers"][0].update(type="other"), "layers[0].type", "other") == 1
    assert bad(lambda c: layer(c, 0).update(tau=0), "tau") == 1
    assert bad(lambda c: layer(c, 3).update(dim=1000), "layers[3]", "dim") == 1
    assert bad(lambda c: layer(c, 1)["rot"].update(dims=4), "rot.dims") == 1
    assert bad(lambda c: layer(c, 1).pop("scale"), "scale") == 1
    assert bad(lambda c: layer(c, 2).update(kv_from=2), "kv_from") == 1
    assert bad(lambda c: layer(c, 2).update(kv_from=0), "kv_from") == 1
    assert bad(lambda c: layer(c, 2).update(kv_rank=9), "kv_from") == 1
    assert bad(lambda c: layer(c, 2)["rot"].update(base=3.0), "kv_from") == 1
    assert bad(lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "mlp.kind") == 1
    assert bad(lambda c: router(c).update(top=7), "router.top") == 1
    assert bad(lambda c: router(c)["groups"].update(count=4), "groups.count") == 1
    assert bad(lambda c: router(c).update(top=3), "groups.keep") == 1
    assert bad(lambda c: None, "l0.mix.a1", drop="l0.mix.a1") == 2
    assert bad(lambda c: None, "l1.mlp.e3.up", drop="l1.mlp.e3.up") == 2
    assert bad(lambda c: None, "l1.mix.sink", drop="l1.mix.sink") == 2
    assert bad(lambda c: None, "side.embed", "shape", shapes="side.embed") == 2
    assert bad(lambda c: None, "l0.mix.a2", "shape", shapes="l0.mix.a1") == 2
