"""The building blocks of the Tudasun layers one by one, each against its plain statement, in both number formats and at
awkward sizes: products with gated pairs, biases, batches and token lists, states that decay per channel, latent attention,
routers with groups, the end of a sublayer, PolyNorm.  Inputs are made so that a mistake shows."""
import ctypes

import numpy as np
import pytest

import kugilix_model as km
import tudasun_plain as plain
from test_gpu_layers import FORMATS, Device, limit

pytestmark = pytest.mark.gpu


@pytest.fixture
def dev(torch_gpu):
    return Device(torch_gpu)


def up(v, m):
    return (v + m - 1) // m * m


class Products:
    """weight blocks and their products"""

    def __init__(self, awq, lib, dev, f32):
        self.awq, self.lib, self.dev, self.f32 = awq, lib, dev, f32

    def block(self, rows, k):
        return self.dev.torch.zeros(self.lib.awq_dense_weight_bytes(rows, k, self.f32), dtype=self.dev.torch.uint8, device="cuda")

    def pack(self, w, block, k, row0, form=0, offset=0):
        d, _ = self.dev.act(w, False)
        self.awq.check(self.lib.awq_dense_pack_form(d.data_ptr(), 0, w.shape[0], w.shape[1], block.data_ptr() + offset, k, row0, 0, form,
                                                    self.f32, self.dev.stream))
        self.dev.torch.cuda.synchronize()

    def run(self, a):
        self.awq.check(self.lib.awq_dense(ctypes.byref(a), self.f32, self.dev.stream))

    def matrix(self, rng, rows, cols, scale=1.0):
        return km.bf16(scale * rng.standard_normal((rows, cols)) / cols ** 0.5)


@pytest.fixture(params=FORMATS, ids=["bf16", "f32"])
def products(request, awq, lib, dev):
    return Products(awq, lib, dev, request.param)


@pytest.mark.parametrize("tokens", [1, 2, 33, 65, 130, 300])
@pytest.mark.parametrize("k", [40, 700])
def test_segments_of_one_input(products, awq, dev, tokens, k):
    """every kind of segment behind one input, at multiples of 32 rows"""
    f32 = products.f32
    print("segments", tokens, k, f32, flush=True)
    rng = np.random.default_rng(tokens + k)
    kp = up(k, 64)
    sizes = {"plain": 37, "sigmoid": 70, "glu": 45, "decay": 33, "forget": 64, "gelu": 21, "one": 1}
    rows0, at = {}, 0
    for n, r in sizes.items():
        rows0[n] = at
        at = up(at + (2 * up(r, 8) if n == "glu" else r), 32)
    block = products.block(up(at, 256), kp)
    w = {n: products.matrix(rng, r, k, 2.0) for n, r in sizes.items()}
    gate = products.matrix(rng, sizes["glu"], k, 2.0)
    for n, m in w.items():
        products.pack(m, block, kp, rows0[n], 2 if n == "glu" else 0)
    products.pack(gate, block, kp, rows0["glu"], 1)
    x, xv = dev.act(np.pad(rng.standard_normal((tokens, k)), ((0, 0), (0, kp - k))), f32)
    xv = xv[:, :k]
    bias = {n: rng.standard_normal(r).astype(np.float32) for n, r in sizes.items()}
    lower = rng.random(sizes["forget"]).astype(np.float32)
    mul, mulv = dev.act(rng.standard_normal((tokens, sizes["gelu"] + 5)), f32)
    z = {n: xv @ m.T for n, m in w.items()}
    g = xv @ gate.T
    want = {"plain": z["plain"], "sigmoid": plain.sigmoid(z["sigmoid"] + bias["sigmoid"]), "glu": plain.silu(g) * z["glu"],
            "decay": -0.3 * np.log1p(np.exp(-(z["decay"] + bias["decay"]))),
            "forget": (1 - lower) * plain.sigmoid(-(z["forget"] + bias["forget"])),
            "gelu": plain.gelu_tanh(z["gelu"]) * mulv[:, :sizes["gelu"]], "one": z["one"]}
    act = {"plain": awq.ACT_NONE, "sigmoid": awq.ACT_SIGMOID, "glu": awq.ACT_GLU, "decay": awq.ACT_LOG_DECAY, "forget": awq.ACT_FORGET,
           "gelu": awq.ACT_GELU, "one": awq.ACT_NONE}
    wide = ("decay", "forget", "one")
    y = {n: dev.empty((tokens, r + (3 if n == "plain" else 0)), f32 or n in wide) for n, r in sizes.items()}
    d_bias = {n: dev.f(b) for n, b in bias.items()}
    d_lower, ws = dev.f(lower), dev.empty((1 << 22,), True)
    a = awq.AwqDenseArgs()
    a.w, a.k, a.tokens, a.n_segments, a.out = block.data_ptr(), kp, tokens, len(sizes), awq.DENSE_STORE
    for i, (n, r) in enumerate(sizes.items()):
        s = awq.AwqDenseSegment(x.data_ptr(), y[n].data_ptr(), kp, y[n].shape[1], rows0[n], 2 * up(r, 8) if n == "glu" else r, act[n])
        s.act_pos, s.y_f32, s.glu_rows = 0.3, n in wide, r if n == "glu" else 0
        s.bias, s.lower = d_bias[n].data_ptr(), d_lower.data_ptr() if n == "forget" else None
        if n == "gelu":
            s.mul, s.ldmul = mul.data_ptr(), mul.shape[1]
        a.segment[i] = s
    for workspace in (0, ws.numel()):  # cut along k or not
        a.workspace, a.workspace_floats = ws.data_ptr(), workspace
        products.run(a)
        for n, r in sizes.items():
            got = dev.host(y[n])
            tight = 2e-5 if f32 or n in wide else 0.012
            assert np.abs(got[:, :r] - want[n]).max() < tight * max(1.0, np.abs(want[n]).max()), n
            assert np.isnan(got[:, r:]).all(), n


def test_softcap(products, awq, dev):
    rng = np.random.default_rng(0)
    w = products.matrix(rng, 50, 64, 6.0)
    block = products.block(256, 64)
    products.pack(w, block, 64, 0)
    for tokens in (1, 40):
        x, xv = dev.act(rng.standard_normal((tokens, 64)), products.f32)
        y = dev.empty((tokens, 50), True)
        a = awq.AwqDenseArgs()
        a.w, a.k, a.tokens, a.n_segments, a.out = block.data_ptr(), 64, tokens, 1, awq.DENSE_F32
        a.segment[0] = awq.AwqDenseSegment(x.data_ptr(), y.data_ptr(), 64, 50, 0, 50, awq.ACT_SOFTCAP, 0, 4.0)
        products.run(a)
        assert np.abs(dev.host(y) - 4 * np.tanh(xv @ w.T / 4)).max() < 2e-5


@pytest.mark.parametrize("tokens", [1, 3, 70, 200])
def test_batches(products, awq, dev, tokens):
    """several products in one launch; for one token also by number, with numbers that are left out"""
    f32 = products.f32
    rng = np.random.default_rng(tokens)
    n, rows, k = 5, 70, 100
    kp, rp = up(k, 64), 256
    size = rp * kp
    block = products.block(n * rp, kp)
    w = [products.matrix(rng, rows, k) for _ in range(n)]
    for i, m in enumerate(w):
        products.pack(m, block, kp, i * rp)
    x, xv = dev.act(np.pad(rng.standard_normal((tokens, n, k)), ((0, 0), (0, 0), (0, kp - k))), f32)
    y = dev.empty((tokens, n, rows), f32)
    a = awq.AwqDenseArgs()
    a.w, a.k, a.tokens, a.n_segments, a.out = block.data_ptr(), kp, tokens, 1, awq.DENSE_STORE
    a.segment[0] = awq.AwqDenseSegment(x.data_ptr(), y.data_ptr(), n * kp, n * rows, 0, rows)
    a.batch, a.w_batch, a.x_batch, a.y_batch = n, size, kp, rows
    products.run(a)
    want = np.stack([xv[:, i, :k] @ w[i].T for i in range(n)], axis=1)
    assert km.rms_error(dev.host(y), want) < limit(f32)
    if tokens == 1:
        ids = [3, 7, 0, 3, 5]
        d_ids = dev.torch.tensor(ids, dtype=dev.torch.int32).cuda()
        y = dev.empty((n, rows), f32)
        a.segment[0].y, a.ids, a.n_groups = y.data_ptr(), d_ids.data_ptr(), n
        products.run(a)
        got = dev.host(y)
        for i, e in enumerate(ids):
            if e < n:
                assert km.rms_error(got[i], xv[0, i, :k] @ w[e].T) < limit(f32)
            else:
                assert np.isnan(got[i]).all()


def route_inputs(rng, tokens, outputs):
    return 2 * rng.standard_normal((tokens, outputs)).astype(np.float32), (0.3 * rng.standard_normal(outputs) - 0.5).astype(np.float32)


ROUTERS = [(8, 8, 2, 0, 0), (10, 8, 4, 2, 1), (12, 9, 3, 4, 2), (6, 6, 6, 0, 0), (70, 64, 5, 7, 3), (300, 290, 8, 10, 4), (4, 0, 2, 2, 1),
           (9, 5, 1, 9, 2)]


@pytest.mark.parametrize("outputs,experts,top,groups,keep", ROUTERS)
@pytest.mark.parametrize("corrected", [True, False])
def test_router(awq, lib, dev, outputs, experts, top, groups, keep, corrected):
    """choice scores are negative throughout: an output that is left out counts as minus infinity, not as 0"""
    print("router", outputs, experts, top, groups, keep, flush=True)
    rng = np.random.default_rng(outputs)
    t = dev.torch
    for tokens, size in ((1, 64), (2, 64), (67, 64), (500, 128), (1500, 64)):
        z, corr = route_inputs(rng, tokens, outputs)
        ld = outputs + 3
        d_z, d_c = dev.f(np.pad(z, ((0, 0), (0, 3)), constant_values=50.0)), dev.f(corr)
        ids = t.full((tokens, top), -1, dtype=t.int32, device="cuda")
        weights = dev.empty((tokens, top), True)
        n_tiles = lib.awq_route_max_tiles(tokens, top, experts, size)
        tiles = t.full((n_tiles, 3), -1, dtype=t.int32, device="cuda")
        lst = t.full((tokens * top,), -1, dtype=t.int32, device="cuda")
        awq.check(lib.awq_route(d_z.data_ptr(), ld, d_c.data_ptr() if corrected else None, outputs, experts, top, groups, keep, tokens,
                                ids.data_ptr(), weights.data_ptr(), size, tiles.data_ptr(), lst.data_ptr(), dev.stream))
        t.cuda.synchronize()
        got_i, got_w = ids.cpu().numpy(), weights.cpu().numpy()
        for i in range(tokens):
            want = plain.choose(z[i].astype(np.float64), corr.astype(np.float64) if corrected else None, top,
                                {"count": groups, "keep": keep} if groups else None)
            assert got_i[i].tolist() == [e for e, _ in want], i
            assert np.allclose(got_w[i], [x for _, x in want], rtol=2e-5)
        if tokens == 1 or experts == 0:
            continue
        # the plan: every entry of an expert once, in runs of one expert
        seen = []
        flat = got_i.reshape(-1)
        for e, first, count in tiles.cpu().numpy():
            assert 0 <= count <= size
            run = lst.cpu().numpy()[first:first + count] if count else []
            assert all(flat[p] == e for p in run)
            seen += list(run)
        assert sorted(seen) == np.flatnonzero(flat < experts).tolist()


@pytest.mark.parametrize("tokens", [2, 40, 300, 700])
def test_products_of_token_lists(products, awq, lib, dev, tokens):
    """a gated product that reads a token per entry and one that reads an entry's own row"""
    f32, t = products.f32, dev.torch
    print("lists", tokens, f32, flush=True)
    rng = np.random.default_rng(tokens)
    experts, outputs, top, width, ff = 6, 8, 3, 72, 45
    size = 128 if tokens == 700 and not f32 else 64
    wk, fk, gu_rows = up(width, 64), up(ff, 64), 256
    gate, upw, down = ([products.matrix(rng, r, c, 1.5) for _ in range(experts)] for r, c in ((ff, width), (ff, width), (width, ff)))
    w_in, w_out = products.block(experts * gu_rows, wk), products.block(experts * 256, fk)
    for e in range(experts):
        products.pack(gate[e], w_in, wk, e * gu_rows, 1)
        products.pack(upw[e], w_in, wk, e * gu_rows, 2)
        products.pack(down[e], w_out, fk, e * 256)
    x, xv = dev.act(np.pad(rng.standard_normal((tokens, width)), ((0, 0), (0, wk - width))), f32)
    z, corr = route_inputs(rng, tokens, outputs)
    d_z, d_c = dev.f(z), dev.f(corr)
    ids, weights = t.zeros((tokens, top), dtype=t.int32, device="cuda"), dev.empty((tokens, top), True)
    n_tiles = lib.awq_route_max_tiles(tokens, top, experts, size)
    tiles, lst = t.zeros((n_tiles, 3), dtype=t.int32, device="cuda"), t.zeros(tokens * top, dtype=t.int32, device="cuda")
    awq.check(lib.awq_route(d_z.data_ptr(), outputs, d_c.data_ptr(), outputs, experts, top, 0, 0, tokens, ids.data_ptr(),
                            weights.data_ptr(), size, tiles.data_ptr(), lst.data_ptr(), dev.stream))
    mid, y = dev.empty((tokens * top, fk), f32, 0.0), dev.empty((tokens * top, width), True)
    a = awq.AwqDenseArgs()
    a.w, a.k, a.tokens, a.n_segments, a.out = w_in.data_ptr(), wk, tokens, 1, awq.DENSE_STORE
    a.segment[0] = awq.AwqDenseSegment(x.data_ptr(), mid.data_ptr(), wk, fk, 0, 2 * up(ff, 8), awq.ACT_GLU)
    a.segment[0].glu_rows = ff
    a.w_batch, a.tiles, a.list, a.max_tiles, a.tile_tokens, a.list_div = gu_rows * wk, tiles.data_ptr(), lst.data_ptr(), n_tiles, size, top
    products.run(a)
    b = awq.AwqDenseArgs()
    b.w, b.k, b.tokens, b.n_segments, b.out = w_out.data_ptr(), fk, tokens, 1, awq.DENSE_STORE
    b.segment[0] = awq.AwqDenseSegment(mid.data_ptr(), y.data_ptr(), fk, width, 0, width)
    b.segment[0].y_f32 = 1
    b.w_batch, b.tiles, b.list, b.max_tiles, b.tile_tokens, b.list_div = 256 * fk, tiles.data_ptr(), lst.data_ptr(), n_tiles, size, 1
    products.run(b)
    got, chosen = dev.host(y), ids.cpu().numpy().reshape(-1)
    scale = 0.0
    for p, e in enumerate(chosen):
        if e >= experts:
            assert np.isnan(got[p]).all()
            continue
        h = xv[p // top, :width]
        want = (plain.silu(h @ gate[e].T) * (h @ upw[e].T)) @ down[e].T
        scale = max(scale, np.abs(want).max())
        assert np.abs(got[p] - want).max() < limit(f32) * max(1.0, scale)


def state_inputs(rng, T, heads, dim, vdim, keys):
    q, v = rng.standard_normal((T, heads, dim)), rng.standard_normal((T, heads, vdim))
    k = rng.standard_normal((T, heads, dim)) if keys else None
    # heads differ: one remembers, one forgets at once, one is mixed, with decays beyond binary32's range between
    rate = np.array([1e-4, 3.0, 0.05, 0.4])[np.arange(heads) % 4][None, :, None] * (0.5 + rng.random((T, heads, dim)))
    if heads > 1:
        rate[T // 3, 1] = 90.0
        rate[T // 2:T // 2 + 40, 1, :dim // 2] = 25.0
    return q, k, v, rate  # decay = 2^-rate


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
@pytest.mark.parametrize("keys", [True, False], ids=["keys", "no keys"])
@pytest.mark.parametrize("heads,dim,vdim", [(3, 20, 12), (4, 64, 64), (2, 128, 96), (2, 256, 40), (3, 101, 35), (2, 300, 16), (4, 9, 31),
                                            (2, 200, 8)])
def test_gated_state(awq, lib, dev, f32, keys, heads, dim, vdim):
    """portions of every form: token by token, full, ragged and single-token chunks"""
    print("gated state", heads, dim, vdim, f32, keys, flush=True)
    rng = np.random.default_rng(dim)
    T = 300
    q, k, v, rate = state_inputs(rng, T, heads, dim, vdim, keys)
    parts = [q.reshape(T, -1)] + ([k.reshape(T, -1)] if keys else []) + [v.reshape(T, -1)]
    n = sum(p.shape[1] for p in parts)
    ldp = up(n, 8)
    proj, pv = dev.act(np.pad(np.concatenate(parts, axis=1), ((0, 0), (0, ldp - n))), f32)
    hd = heads * dim
    qv = pv[:, :hd].reshape(T, heads, dim)
    vv = pv[:, n - heads * vdim:n].reshape(T, heads, vdim)
    if keys:
        g = (-rate).astype(np.float32)
        decay, kv = 2.0 ** g.astype(np.float64), pv[:, hd:2 * hd].reshape(T, heads, dim)
    else:
        g = (1.0 - 2.0 ** -rate).astype(np.float32)
        g[T // 4, 0, :] = 1.0  # a decay of exactly zero
        kv = g.astype(np.float64)
        decay = 1.0 - kv
    want, S = plain.gated_state(qv * 0.3, kv, vv, decay)
    d_g = dev.f(g.reshape(T, hd))
    dimp = up(dim, 64)
    for sizes in ([300], [1], [2, 15], [16], [17, 1, 2], [64], [130, 31]):
        state = dev.empty((heads, vdim, dimp), True)  # NaN: position 0 starts from nothing
        out, at, i = [], 0, 0
        while at < T:
            m = min(sizes[i % len(sizes)], T - at)
            o = dev.empty((m, heads * vdim), True)
            base = proj[at:].data_ptr()
            unit = proj.element_size()
            a = awq.AwqGatedStateArgs(base, base + hd * unit if keys else None, base + (n - heads * vdim) * unit, d_g[at:].data_ptr(),
                                      ldp, hd, heads, dim, vdim, 0.3, state.data_ptr(), o.data_ptr(), m, at)
            awq.check(lib.awq_gated_state(ctypes.byref(a), f32, dev.stream))
            out.append(o)
            at, i = at + m, i + 1
        got = dev.host(dev.torch.cat(out)).reshape(T, heads, vdim)
        for h in range(heads):  # per head: a head that forgets at once is small beside one that remembers
            assert km.rms_error(got[:, h], want[:, h]) < 5e-5, (sizes, h)
        s = dev.host(state)[:, :, :dim].transpose(0, 2, 1)
        for h in range(heads):
            assert np.abs(s[h] - S[h]).max() <= 5e-5 * np.abs(S[h]).max(), (sizes, h)


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
def test_a_key_far_back_in_a_state(awq, lib, dev, f32):
    """one token writes a marked row, hundreds of tokens later a query reads just that row"""
    T, dim, vdim, far = 420, 64, 32, 37
    q, k, v = np.zeros((T, 1, dim)), np.zeros((T, 1, dim)), np.random.default_rng(2).standard_normal((T, 1, vdim))
    k[:, 0, 1:] = 1.0
    k[far, 0] = np.eye(1, dim)[0]
    q[:, 0, 0] = 1.0
    g = np.full((T, dim), -0.002, np.float32)
    proj, pv = dev.act(np.concatenate([x.reshape(T, -1) for x in (q, k, v)], axis=1), f32)
    d_g = dev.f(g)
    want, _ = plain.gated_state(q, k, pv[:, 2 * dim:].reshape(T, 1, vdim), 2.0 ** g.astype(np.float64).reshape(T, 1, dim))
    assert np.abs(want[far - 1]).max() == 0 and np.abs(want[-1]).max() > 0.5
    for sizes in ([T], [far], [far + 1], [64, 1], [1]):
        state = dev.empty((1, vdim, 64), True)
        at, i, out = 0, 0, []
        while at < T:
            m = min(sizes[i % len(sizes)], T - at)
            o, base, unit = dev.empty((m, vdim), True), proj[at:].data_ptr(), proj.element_size()
            a = awq.AwqGatedStateArgs(base, base + dim * unit, base + 2 * dim * unit, d_g[at:].data_ptr(), proj.shape[1], dim, 1, dim,
                                      vdim, 1.0, state.data_ptr(), o.data_ptr(), m, at)
            awq.check(lib.awq_gated_state(ctypes.byref(a), f32, dev.stream))
            out.append(o)
            at, i = at + m, i + 1
        assert np.abs(dev.host(dev.torch.cat(out)) - want[:, 0]).max() < 1e-5 * np.abs(want).max(), sizes


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
@pytest.mark.parametrize("heads,dim,vdim", [(3, 20, 12), (2, 128, 128), (5, 70, 33), (1, 320, 520)])
@pytest.mark.parametrize("gated", [True, False])
def test_head_norm_alone_and_behind_a_step(awq, lib, dev, f32, heads, dim, vdim, gated):
    rng = np.random.default_rng(vdim)
    n, hd = heads * vdim, heads * dim
    w, eps = 1 + 0.3 * rng.standard_normal(vdim).astype(np.float32), 1e-3
    d_w = dev.f(w)
    o = 3 * rng.standard_normal((7, n)).astype(np.float32)
    gate, gv = dev.act(2 * rng.standard_normal((7, n + 3)), f32)
    ctx, d_o = dev.empty((7, n + 5), f32), dev.f(o)
    awq.check(lib.awq_head_norm(d_o.data_ptr(), gate.data_ptr() if gated else None, n + 3, d_w.data_ptr(), ctx.data_ptr(), n + 5, heads,
                                vdim, 7, eps, f32, dev.stream))
    finish = lambda x, g: (plain.rms(x, eps) * w).reshape(-1, n) * (plain.silu(g) if gated else 1.0)
    want = finish(o.astype(np.float64).reshape(7, heads, vdim), gv[:, :n])
    got = dev.host(ctx)
    assert km.rms_error(got[:, :n], want) < (2e-6 if f32 else 0.006) and np.isnan(got[:, n:]).all()
    # one token: recurrence, norm and gate in one launch
    T = 4
    q, k, v, rate = state_inputs(rng, T, heads, dim, vdim, True)
    proj, pv = dev.act(np.concatenate([x.reshape(T, -1) for x in (q, k, v)], axis=1), f32)
    d_g = dev.f(-rate.reshape(T, hd))
    ref, _ = plain.gated_state(pv[:, :hd].reshape(T, heads, dim), pv[:, hd:2 * hd].reshape(T, heads, dim),
                               pv[:, 2 * hd:].reshape(T, heads, vdim), 2.0 ** -rate.astype(np.float32).astype(np.float64))
    state = dev.empty((heads, vdim, up(dim, 64)), True)
    for t in range(T):
        c, base, unit = dev.empty((n,), f32), proj[t:].data_ptr(), proj.element_size()
        a = awq.AwqGatedStateArgs(base, base + hd * unit, base + 2 * hd * unit, d_g[t:].data_ptr(), proj.shape[1], hd, heads, dim, vdim, 1.0,
                                  state.data_ptr(), None, 1, t, d_w.data_ptr(), gate.data_ptr() if gated else None, c.data_ptr(), eps)
        awq.check(lib.awq_gated_state(ctypes.byref(a), f32, dev.stream))
        want = finish(ref[t:t + 1], gv[:1, :n])
        assert km.rms_error(dev.host(c)[None], want) < (3e-5 if f32 else 0.006), t


class Latent:
    """one layer of latent attention: weights, cache and scratch"""

    def __init__(self, awq, lib, dev, f32, heads, dim, rot, vdim, rank, uk, uv, norm, sink, scale, eps, base, max_pos, max_tokens, cache=None):
        self.awq, self.lib, self.dev, self.f32 = awq, lib, dev, f32
        torch = dev.torch
        self.row = lib.awq_latent_row(rank, rot)
        a = self.a = awq.AwqLatentArgs()
        a.heads, a.dim, a.vdim, a.rank, a.rot, a.scale, a.eps, a.max_pos = heads, dim, vdim, rank, rot, scale, eps, max_pos
        need = awq.AwqLatentBytes()
        awq.check(lib.awq_latent_sizes(ctypes.byref(a), max_tokens, f32, ctypes.byref(need)))
        self.forms = need.w_kv > 0
        self.cache = cache if cache is not None else dev.empty((up(max_pos, 64), self.row), f32, 0.0)
        zeros = lambda n: torch.zeros(max(4, n), dtype=torch.uint8, device="cuda")
        self.keep = {n: zeros(getattr(need, n)) for n, _ in need._fields_}
        for n, t in self.keep.items():
            setattr(a, n, t.data_ptr() if getattr(need, n) else None)
        self.norm, self.sink = dev.f(norm), dev.f(sink) if sink is not None else None
        self.freq = torch.tensor([base ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=torch.float64).cuda()
        a.norm, a.freq, a.sink, a.cache = self.norm.data_ptr(), self.freq.data_ptr(), self.sink.data_ptr() if sink is not None else None, \
            self.cache.data_ptr()
        k, v = dev.act(uk, False)[0], dev.act(uv, False)[0]
        awq.check(lib.awq_latent_pack(ctypes.byref(a), k.data_ptr(), v.data_ptr(), f32, dev.stream))
        torch.cuda.synchronize()

    def run(self, q, down, pos0):
        a, n = self.a, q.shape[0]
        ldq = up(q.shape[1], 8)
        x = self.dev.act(np.pad(q, ((0, 0), (0, ldq - q.shape[1]))), self.f32)[0]
        d = self.dev.f(down) if down is not None else None
        ldc = up(a.heads * a.vdim, 64)
        ctx = self.dev.empty((n, ldc), self.f32)
        a.q, a.ldq, a.down, a.ldd = x.data_ptr(), ldq, d.data_ptr() if d is not None else None, a.rank + a.rot
        a.ctx, a.ldc, a.n_tokens, a.pos0 = ctx.data_ptr(), ldc, n, pos0
        self.awq.check(self.lib.awq_latent_attention(ctypes.byref(a), self.f32, self.dev.stream))
        return self.dev.host(ctx)[:, :a.heads * a.vdim].reshape(n, a.heads, a.vdim)


def portions(T, sizes):
    at, i = 0, 0
    while at < T:
        n = min(sizes[i % len(sizes)], T - at)
        yield at, n
        at, i = at + n, i + 1


LATENTS = [(3, 20, 6, 12, 37), (4, 64, 32, 64, 128), (40, 16, 16, 24, 64), (2, 128, 64, 128, 512), (1, 72, 2, 40, 300), (2, 8, 8, 256, 200),
           (2, 192, 64, 64, 96), (1, 100, 30, 20, 700)]


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
@pytest.mark.parametrize("shape", LATENTS, ids=str)
def test_latent_attention(awq, lib, dev, f32, shape):
    """whole prompts, portions and single tokens over several tiles of the cache; a second layer on the same rows"""
    heads, dim, rot, vdim, rank = shape
    print("latent attention", shape, f32, flush=True)
    rng = np.random.default_rng(rank)
    T, eps, base, scale = 330, 1e-3, 300.0, 2.5 * (dim + rot) ** -0.5
    q = km.bf16(rng.standard_normal((T, heads * (dim + rot))))
    down = rng.standard_normal((T, rank + rot)).astype(np.float32)
    norm, sink = 1 + 0.3 * rng.standard_normal(rank), 2 * rng.standard_normal(heads)
    uk, uv = (km.bf16(rng.standard_normal((heads * n, rank)) / rank ** 0.5) for n in (dim, vdim))
    c = plain.rms(down[:, :rank].astype(np.float64), eps) * norm.astype(np.float32)
    kr = plain.rotate(down[:, rank:].astype(np.float64), 0, base)
    qh = q.reshape(T, heads, dim + rot).astype(np.float64)
    want = plain.latent_attention(qh[:, :, :dim], plain.rotate(qh[:, :, dim:], 0, base), c, kr, uk.reshape(heads, dim, rank),
                                  uv.reshape(heads, vdim, rank), scale, sink)
    layer = Latent(awq, lib, dev, f32, heads, dim, rot, vdim, rank, uk, uv, norm, sink, scale, eps, base, T, T)
    for sizes in ([T], [1], [2, 63, 1], [200, 1], [64, 65], [31]):
        if sizes == [1] and rank > 600:
            continue
        got = np.concatenate([layer.run(q[at:at + n], down[at:at + n], at) for at, n in portions(T, sizes)])
        assert km.rms_error(got, want) < (3e-5 if f32 else 0.03), sizes
    # another layer with heads, weights and sinks of its own on these rows
    other = Latent(awq, lib, dev, f32, heads + 1, dim, rot, vdim, rank, np.concatenate([uk, uk[:dim]]), np.concatenate([uv[:vdim], uv]), norm,
                   None, 0.5 * scale, eps, base, T, T, cache=layer.cache)
    q2 = km.bf16(rng.standard_normal((T, (heads + 1) * (dim + rot))))
    qh = q2.reshape(T, heads + 1, dim + rot).astype(np.float64)
    want = plain.latent_attention(qh[:, :, :dim], plain.rotate(qh[:, :, dim:], 0, base), c, kr,
                                  np.concatenate([uk, uk[:dim]]).reshape(-1, dim, rank), np.concatenate([uv[:vdim], uv]).reshape(-1, vdim, rank),
                                  0.5 * scale, None)
    for sizes in ([T], [130, 1, 2]):
        got = np.concatenate([other.run(q2[at:at + n], None, at) for at, n in portions(T, sizes)])
        assert km.rms_error(got, want) < (3e-5 if f32 else 0.03), sizes


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
@pytest.mark.parametrize("shape", [(2, 64, 32, 64, 128), (3, 20, 6, 12, 37)], ids=str)
def test_a_key_far_back_and_the_sink(awq, lib, dev, f32, shape):
    """One key outweighs all others wherever it lies (the first position, the borders of tiles of 64), for every later query
    and for none before it; without it the sink takes the weight and the output all but vanishes."""
    heads, dim, rot, vdim, rank = shape
    rng = np.random.default_rng(1)
    T, scale, base = 400, 1.0, 10.0
    uk, uv = np.zeros((heads * dim, rank)), km.bf16(rng.standard_normal((heads * vdim, rank)))
    uk.reshape(heads, dim, rank)[:, 0, 0] = 1.0                # the first unrotated entry is the first latent
    q = np.zeros((T, heads, dim + rot), np.float32)
    q[:, :, 0] = 4.0
    sink = np.full(heads, 8.0)
    for far in (0, 1, 63, 64, 127, 128, 255, 319):
        down = 0.1 * rng.standard_normal((T, rank + rot)).astype(np.float32)
        down[:, 0] = 0.0
        down[far, :rank] = 0.0
        down[far, 0] = 1.0                                      # after the norm: sqrt(rank) in one place
        c = plain.rms(down[:, :rank].astype(np.float64), 1e-6)
        want = plain.latent_attention(q[:, :, :dim].astype(np.float64), q[:, :, dim:].astype(np.float64) * 0, c,
                                      plain.rotate(down[:, rank:].astype(np.float64), 0, base), uk.reshape(heads, dim, rank),
                                      uv.reshape(heads, vdim, rank), scale, sink)
        norm = np.ones(rank)
        size = np.abs(want[far:]).max()
        layer = Latent(awq, lib, dev, f32, heads, dim, rot, vdim, rank, uk, uv, norm, sink, scale, 1e-6, base, T, T)
        assert far == 0 or np.abs(want[:far]).max() < 0.5 * size
        for sizes in ([T], [63], [150, 1, 1, 2], [1]):
            if sizes == [1] and far not in (0, 64):
                continue
            got = np.concatenate([layer.run(q.reshape(T, -1)[at:at + n], down[at:at + n], at) for at, n in portions(T, sizes)])
            assert np.abs(got - want).max() < (1e-4 if f32 else 0.012) * size, (far, sizes)


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
@pytest.mark.parametrize("width", [32, 90, 1024, 5001])
def test_the_end_of_a_sublayer(awq, lib, dev, f32, width):
    rng = np.random.default_rng(width)
    eps, top, experts = 1e-3, 3, 4
    for T in (1, 5, 600):
        if T == 600 and width > 1024:
            continue
        x, y = rng.standard_normal((2, T, width)).astype(np.float32)
        w1, w2 = (1 + 0.3 * rng.standard_normal((2, width))).astype(np.float32)
        ld = up(width, 8)
        gate, gv = dev.act(rng.random((T, ld)), f32)
        h, hv = dev.act(rng.standard_normal((T, ld)), f32)
        sg, pairs = rng.standard_normal(T).astype(np.float32), rng.standard_normal((T * top, width)).astype(np.float32)
        ids = rng.integers(0, experts + 2, (T, top)).astype(np.int32)
        pairs[ids.reshape(-1) >= experts] = np.nan   # not read
        weights = rng.random((T, top)).astype(np.float32)
        d = {n: dev.f(v) for n, v in dict(y=y, w1=w1, w2=w2, sg=sg, pairs=pairs, weights=weights).items()}
        d_ids = dev.torch.from_numpy(ids).cuda()
        routed = np.zeros((T, width))
        for t in range(T):
            for j in range(top):
                routed[t] += weights[t, j] * (pairs[t * top + j].astype(np.float64) if ids[t, j] < experts else hv[t, :width])
        for dense, moe, gated, norm in ((1, 0, 1, 1), (1, 0, 0, 0), (1, 1, 1, 0), (0, 1, 1, 1)):
            s = np.zeros((T, width))
            a = awq.AwqJoinArgs()
            dx, out = dev.f(x), dev.empty((T, ld), f32)
            a.x, a.n_tokens, a.width, a.eps = dx.data_ptr(), T, width, eps
            if dense:
                a.y, s = d["y"].data_ptr(), s + y
            if moe:
                if dense:
                    a.y_gate, s = d["sg"].data_ptr(), s * plain.sigmoid(sg.astype(np.float64))[:, None]
                a.pairs, a.ids, a.weights, a.h, a.ldh = d["pairs"].data_ptr(), d_ids.data_ptr(), d["weights"].data_ptr(), h.data_ptr(), ld
                a.top, a.experts, s = top, experts, s + routed
            if gated:
                a.gate, a.ldg, s = gate.data_ptr(), ld, s * gv[:, :width]
            a.w_post, a.out, a.ldo = d["w1"].data_ptr(), out.data_ptr(), ld
            if norm:
                a.w_next = d["w2"].data_ptr()
            awq.check(lib.awq_join(ctypes.byref(a), f32, dev.stream))
            want = x + plain.rms(s, eps) * w1
            assert np.abs(dev.host(dx) - want).max() < 2e-5
            want = plain.rms(want, eps) * w2 if norm else want
            got = dev.host(out)
            assert np.all(np.abs(got[:, :width] - want) <= (3e-5 if f32 else 0.004 * np.abs(want) + 1e-3)) and np.isnan(got[:, width:]).all()


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
@pytest.mark.parametrize("n", [3, 64, 333, 12288])
def test_polynorm(awq, lib, dev, f32, n):
    rng = np.random.default_rng(n)
    abce = np.array([0.7, -1.3, 0.4, 0.25], np.float32)
    for T in (1, 9, 520):
        if T == 520 and n > 333:
            continue
        z, zv = dev.act(3 * rng.standard_normal((T, n + 5 - n % 4)), f32)
        d = dev.f(abce)
        awq.check(lib.awq_polynorm(z.data_ptr(), z.shape[1], n, T, d.data_ptr(), 1e-3, f32, dev.stream))
        got = dev.host(z)
        assert km.rms_error(got[:, :n], plain.polynorm(zv[:, :n], abce.astype(np.float64), 1e-3)) < (3e-6 if f32 else 0.006)
        assert np.array_equal(got[:, n:], zv[:, n:])
