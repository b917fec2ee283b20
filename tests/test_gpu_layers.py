"""The layer building blocks one by one (dense products, norms with convolution, window attention, linear attention,
sinusoidal embedding), each against its plain statement, in both number formats and at awkward sizes.  Inputs are made
so that a mistake shows: a key at the very edge of a window outweighs all others, states decay slowly."""
import ctypes

import numpy as np
import pytest

import kugilix_model as km
import kugilix_plain as plain

pytestmark = pytest.mark.gpu

FORMATS = [False, True]  # f32


@pytest.fixture
def dev(torch_gpu):
    return Device(torch_gpu)


class Device:
    def __init__(self, torch):
        self.torch = torch
        self.stream = ctypes.c_void_p(torch.cuda.current_stream().cuda_stream)

    def act(self, x, f32):
        """activations in the format under test; returns (tensor, the values it holds)"""
        x = np.ascontiguousarray(x, np.float32)
        if f32:
            return self.f(x), x.astype(np.float64)
        return self.torch.from_numpy(x).cuda().to(self.torch.bfloat16), km.bf16(x).astype(np.float64)

    def f(self, x):
        return self.torch.from_numpy(np.ascontiguousarray(x, np.float32)).cuda()

    def empty(self, shape, f32, fill=float("nan")):
        return self.torch.full(shape, fill, dtype=self.torch.float32 if f32 else self.torch.bfloat16, device="cuda")

    def host(self, t):
        self.torch.cuda.synchronize()
        return t.float().cpu().numpy().astype(np.float64)


def limit(f32):
    return 2e-5 if f32 else 0.012


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
@pytest.mark.parametrize("tokens", [1, 2, 33, 65, 130, 300])
@pytest.mark.parametrize("shape", [(70, 90, 50), (300, 1536, 520)], ids=str)
def test_dense_two_segments(awq, lib, dev, f32, tokens, shape):
    """[A; B] in one block: silu on part of A's rows, xIELU on B's, each with an input of its own"""
    na, k, nb = shape
    print("dense", shape, tokens, f32, flush=True)
    rng = np.random.default_rng(tokens)
    up = lambda v, m: (v + m - 1) // m * m
    kp, row_b = up(k, 64), up(na, 256)
    rows = row_b + up(nb, 256)
    block = dev.torch.zeros(lib.awq_dense_weight_bytes(rows, kp, f32), dtype=dev.torch.uint8, device="cuda")
    wa, wb = km.bf16(rng.standard_normal((na, k)) / k ** 0.5), km.bf16(2 * rng.standard_normal((nb, k)) / k ** 0.5)
    for w, r0 in ((wa, 0), (wb, row_b)):
        d, _ = dev.act(w, False)
        awq.check(lib.awq_dense_pack(d.data_ptr(), 0, w.shape[0], k, block.data_ptr(), kp, r0, 0, f32, dev.stream))
    pad = lambda x: np.pad(x, ((0, 0), (0, kp - k)))
    xa, va = dev.act(pad(rng.standard_normal((tokens, k))), f32)
    xb, vb = dev.act(pad(rng.standard_normal((tokens, k))), f32)
    ya, yb = dev.empty((tokens, na + 3), f32), dev.empty((tokens, nb), f32)
    ws = dev.empty((1 << 22,), True)
    p, q = 0.4, -0.3
    a = awq.AwqDenseArgs()
    a.w, a.k, a.tokens, a.n_segments, a.out = block.data_ptr(), kp, tokens, 2, awq.DENSE_STORE
    sp = lambda z: float(plain.softplus(np.float64(z)))
    a.segment[0] = awq.AwqDenseSegment(xa.data_ptr(), ya.data_ptr(), kp, na + 3, 0, na, awq.ACT_SILU, na // 2, 0, 0)
    a.segment[1] = awq.AwqDenseSegment(xb.data_ptr(), yb.data_ptr(), kp, nb, row_b, nb, awq.ACT_XIELU, 0, sp(p), 0.5 + sp(q))
    a.workspace, a.workspace_floats = ws.data_ptr(), ws.numel()
    awq.check(lib.awq_dense(ctypes.byref(a), f32, dev.stream))
    za, zb = va[:, :k] @ wa.T, vb[:, :k] @ wb.T
    za[:, :na // 2] = plain.silu(za[:, :na // 2])
    got = dev.host(ya)
    assert km.rms_error(got[:, :na], za) < limit(f32) and np.isnan(got[:, na:]).all()
    assert km.rms_error(dev.host(yb), plain.xielu(zb, p, q)) < limit(f32)
    # residual form, with and without an addend; and as floats
    for addend in (None, rng.standard_normal((tokens, na))):
        y0 = rng.standard_normal((tokens, na))
        y = dev.f(y0)
        ad = dev.f(addend) if addend is not None else None
        a.n_segments, a.out, a.addend = 1, awq.DENSE_RESIDUAL, ad.data_ptr() if ad is not None else None
        a.segment[0] = awq.AwqDenseSegment(xa.data_ptr(), y.data_ptr(), kp, na, 0, na, 0, 0, 0, 0)
        awq.check(lib.awq_dense(ctypes.byref(a), f32, dev.stream))
        assert km.rms_error(dev.host(y), y0 + va[:, :k] @ wa.T + (0 if addend is None else addend)) < 2e-5
    y = dev.empty((tokens, na), True)
    a.out, a.addend = awq.DENSE_F32, None
    a.segment[0] = awq.AwqDenseSegment(xa.data_ptr(), y.data_ptr(), kp, na, 0, na, 0, 0, 0, 0)
    awq.check(lib.awq_dense(ctypes.byref(a), f32, dev.stream))
    assert km.rms_error(dev.host(y), va[:, :k] @ wa.T) < 2e-5


def test_xielu_near_zero_and_far_out(awq, lib, dev):
    """the negative branch cancels near zero: small arguments keep their relative accuracy"""
    z = np.concatenate([-np.geomspace(1e-6, 60, 200), np.geomspace(1e-6, 60, 56)]).astype(np.float32)
    w = dev.torch.zeros(256 * 64, dtype=dev.torch.float32, device="cuda")
    d = dev.f(z.reshape(256, 1))
    awq.check(lib.awq_dense_pack(d.data_ptr(), 1, 256, 1, w.data_ptr(), 64, 0, 0, 1, dev.stream))
    x = dev.f(np.eye(1, 64))
    y = dev.empty((1, 256), True)
    a = awq.AwqDenseArgs()
    a.w, a.k, a.tokens, a.n_segments, a.out = w.data_ptr(), 64, 1, 1, awq.DENSE_STORE
    sp = lambda v: float(plain.softplus(np.float64(v)))
    a.segment[0] = awq.AwqDenseSegment(x.data_ptr(), y.data_ptr(), 64, 256, 0, 256, awq.ACT_XIELU, 0, sp(0.2), 0.5 + sp(1.3))
    awq.check(lib.awq_dense(ctypes.byref(a), 1, dev.stream))
    want = plain.xielu(z.astype(np.float64), 0.2, 1.3)
    # (the function has a zero near -1 / act_neg: there the parts it is the sum of set the scale)
    assert np.all(np.abs(dev.host(y)[0] - want) <= 5e-7 * np.maximum(np.abs(want), np.abs(z)))


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
def test_embedding_with_positions(awq, lib, dev, f32):
    rng = np.random.default_rng(0)
    for width, pos0 in ((7, 0), (96, 3), (130, 70000)):
        table, vals = dev.act(rng.standard_normal((19, width)), f32)
        tokens = rng.integers(0, 19, 33).astype(np.int32)
        freq = dev.torch.tensor([10000.0 ** (-2.0 * i / width) for i in range((width + 1) // 2)], dtype=dev.torch.float64).cuda()
        ids = dev.torch.from_numpy(tokens).cuda()
        x = dev.empty((33, width), True)
        awq.check(lib.awq_embed_sinusoid(table.data_ptr(), f32, ids.data_ptr(), pos0, 33, width, 1.7, freq.data_ptr(),
                                         x.data_ptr(), dev.stream))
        want = plain.embed(tokens, vals, np.float32(1.7), pos0)
        assert np.abs(dev.host(x) - want).max() < 2e-6


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
@pytest.mark.parametrize("width,groups,taps", [(96, 4, 4), (90, 5, 3), (64, 1, 1), (64, 2, 2), (1280, 2, 8), (48, 3, 11), (2048, 1, 4)])
def test_norm_and_convolution_in_portions(awq, lib, dev, f32, width, groups, taps):
    print("norm_conv", width, groups, taps, f32, flush=True)
    rng = np.random.default_rng(width)
    T, eps = 75, 0.03
    x = rng.standard_normal((T, width)).astype(np.float32) * np.linspace(0.1, 3, T, dtype=np.float32)[:, None]
    w1, w2 = 1 + 0.5 * rng.standard_normal(width), rng.standard_normal(width)
    conv = rng.standard_normal((width, taps))
    h = plain.grouped_norm(x.astype(np.float64), w1.astype(np.float32), groups, eps)
    want1, want2 = plain.causal_conv(h, conv.astype(np.float32)), plain.grouped_norm(x.astype(np.float64), w2, groups, eps)
    d_w1, d_w2, d_c = dev.f(w1), dev.f(w2), dev.f(conv)
    ld = width + 8 - width % 8
    for sizes in ([75], [1], [2], [5, 1, 3], [taps, 1], [64, 2]):
        state = [dev.empty((max(1, taps - 1), width), True) for _ in range(2)]  # NaN: nothing ahead of 0 is read
        at, i = 0, 0
        while at < T:
            n = min(sizes[i % len(sizes)], T - at)
            xs = dev.f(x[at:at + n])
            y1, y2 = dev.empty((n, ld), f32), dev.empty((n, ld), f32)
            awq.check(lib.awq_norm_conv(xs.data_ptr(), n, width, groups, eps, d_w1.data_ptr(), d_c.data_ptr(), taps,
                                        state[i & 1].data_ptr(), state[i & 1 ^ 1].data_ptr(), y1.data_ptr(), d_w2.data_ptr(),
                                        y2.data_ptr(), ld, at, f32, dev.stream))
            assert np.abs(dev.host(y1)[:, :width] - want1[at:at + n]).max() <= (1e-5 if f32 else 0.01) * np.abs(want1).max()
            assert np.abs(dev.host(y2)[:, :width] - want2[at:at + n]).max() <= (1e-5 if f32 else 0.01) * np.abs(want2).max()
            at, i = at + n, i + 1


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
@pytest.mark.parametrize("n", [37, 96, 4096, 5000])
def test_gated_norm(awq, lib, dev, f32, n):
    rng = np.random.default_rng(n)
    for T in (1, 9):
        o, w = 4 * rng.standard_normal((T, n)), rng.standard_normal(n)
        ldg = n + 8 - n % 8
        g, gv = dev.act(5 * rng.standard_normal((T, ldg)), f32)
        y = dev.empty((T, ldg), f32)
        d_o, d_w = dev.f(o), dev.f(w)
        awq.check(lib.awq_gated_norm(d_o.data_ptr(), n, g.data_ptr(), ldg, d_w.data_ptr(), y.data_ptr(), ldg, n, T, 1e-3, f32,
                                     dev.stream))
        want = plain.rms(o.astype(np.float32).astype(np.float64), 1e-3) * w * plain.sigmoid(gv[:, :n])
        assert km.rms_error(dev.host(y)[:, :n], want) < (2e-6 if f32 else 0.004)


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
@pytest.mark.parametrize("heads,dim,vdim", [(3, 20, 12), (2, 64, 64), (2, 128, 96), (1, 256, 40), (2, 100, 36), (1, 512, 16),
                                            (4, 9, 31), (1, 200, 8)])
def test_linear_attention(awq, lib, dev, f32, heads, dim, vdim):
    """portions of every form: token by token, chunks that are full, ragged and of one token, several chunks"""
    print("linear attention", heads, dim, vdim, f32, flush=True)
    rng = np.random.default_rng(dim)
    T = 300
    n = heads * (2 * dim + vdim)
    ldp = (n + 7) // 8 * 8
    proj, pv = dev.act(np.pad(rng.standard_normal((T, n)) * 0.5 + 0.2, ((0, 0), (0, ldp - n))), f32)
    q = pv[:, :heads * dim].reshape(T, heads, dim)
    k = pv[:, heads * dim:2 * heads * dim].reshape(T, heads, dim)
    v = pv[:, 2 * heads * dim:n].reshape(T, heads, vdim)
    decay = np.array([0.999, 0.3, 0.9, 1e-6][:heads], np.float32)
    want, S = plain.linear_attention(q, k, v, decay.astype(np.float64))
    d_decay, d_lg = dev.f(decay), dev.f(np.log2(decay.astype(np.float64)))
    dimp = (dim + 63) // 64 * 64
    for sizes in ([300], [1], [2, 15], [16], [129, 1, 2], [128], [130, 31]):
        if f32 and sizes not in ([300], [1], [2, 15]):
            continue
        state = dev.empty((heads, vdim, dimp), True)  # NaN: position 0 starts from nothing
        out, at, i = [], 0, 0
        while at < T:
            m = min(sizes[i % len(sizes)], T - at)
            o = dev.empty((m, heads * vdim), True)
            awq.check(lib.awq_linear_attention(proj[at:].data_ptr(), ldp, heads, dim, vdim, d_decay.data_ptr(), d_lg.data_ptr(),
                                               state.data_ptr(), o.data_ptr(), m, at, f32, dev.stream))
            out.append(o)
            at, i = at + m, i + 1
        got = dev.host(dev.torch.cat(out)).reshape(T, heads, vdim)
        for h in range(heads):  # per head: a head that forgets at once is small beside one that remembers
            # the operands are exact, so both forms carry (nearly) binary32
            assert km.rms_error(got[:, h], want[:, h]) < 3e-5, (sizes, h)
        s = dev.host(state)[:, :, :dim].transpose(0, 2, 1)
        for h in range(heads):
            assert np.abs(s[h] - S[h]).max() <= 3e-5 * np.abs(S[h]).max(), (sizes, h)


def attend(awq, lib, dev, f32, proj, heads, kv, dim, vdim, window, scale, eps, temp, sizes, T, slots, max_pos):
    """the attention of T tokens in portions; proj: the tensor with all tokens' projections (kept as it is)"""
    kr, vr = lib.awq_window_row(dim), lib.awq_window_row(vdim)
    kc, vc = dev.empty((slots, kv, kr), f32, 0.0), dev.empty((slots, kv, vr), f32, 0.0)
    ws = dev.empty((max(1, lib.awq_window_workspace_floats(heads, vdim, window, max_pos)),), True)
    slope = dev.f([plain.slope(h, heads) for h in range(heads)])
    n = heads * vdim
    ldc = (n + 7) // 8 * 8
    out, at, i = [], 0, 0
    while at < T:
        m = min(sizes[i % len(sizes)], T - at)
        p = proj[at:at + m].clone()
        ctx = dev.empty((m, ldc), f32)
        a = awq.AwqWindowArgs(p.data_ptr(), p.shape[1], heads, kv, dim, vdim, window, slots, scale, eps, temp[0], 0, temp[1],
                              slope.data_ptr(), kc.data_ptr(), vc.data_ptr(), ctx.data_ptr(), ldc, m, at, max_pos, ws.data_ptr())
        awq.check(lib.awq_window_attention(ctypes.byref(a), f32, dev.stream))
        dev.torch.cuda.synchronize()
        out.append(ctx)
        at, i = at + m, i + 1
    return dev.host(dev.torch.cat(out))[:, :n].reshape(T, heads, vdim)


SHAPES = [(4, 2, 64, 64), (3, 3, 128, 128), (6, 1, 20, 12), (2, 1, 256, 96), (12, 1, 32, 200), (1, 1, 300, 72), (10, 2, 64, 36)]


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
@pytest.mark.parametrize("shape", SHAPES, ids=str)
@pytest.mark.parametrize("window", [0, 1, 33, 64, 65, 129])
def test_window_attention(awq, lib, dev, f32, shape, window):
    """random scores of some size: prompts, portions and single tokens, over several cache blocks"""
    heads, kv, dim, vdim = shape
    print("window attention", shape, window, f32, flush=True)
    rng = np.random.default_rng(dim + window)
    T, eps, scale, temp = 200, 1e-3, 3.0 / dim ** 0.5, (0.7, 13.0)
    n = heads * dim + kv * (dim + vdim)
    proj, pv = dev.act(np.pad(2 * rng.standard_normal((T, n)), ((0, 0), (0, -n % 8))), f32)
    q = plain.rms(pv[:, :heads * dim].reshape(T, heads, dim), eps)
    k = plain.rms(pv[:, heads * dim:(heads + kv) * dim].reshape(T, kv, dim), eps)
    if not f32:  # what the matrix cores are given
        q, k = km.bf16(q).astype(np.float64), km.bf16(k).astype(np.float64)
    v = pv[:, (heads + kv) * dim:n].reshape(T, kv, vdim)
    want = plain.window_attention(q, k, v, window or None, scale, temp)
    for sizes in ([200], [1], [2, 63, 1], [100, 1]):
        slots = 256 if not window else (window - 1 + max(sizes) + 63) // 64 * 64
        got = attend(awq, lib, dev, f32, proj, heads, kv, dim, vdim, window, scale, eps, temp, sizes, T, slots, T)
        assert km.rms_error(got, want) < (3e-5 if f32 else 0.01), sizes


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 64, 65, 96, 128, 160])
def test_window_edges(awq, lib, dev, f32, window):
    """One key outweighs every other for all queries.  At distance window - 1 it is all a query sees, at distance
    window nothing of it is left; in prompts, portions and decoding, wherever the key lies."""
    print("window edge", window, f32, flush=True)
    heads, kv, dim, vdim = 2, 1, 64, 64
    rng = np.random.default_rng(window)
    T = 330
    for far in (0, 5, 63, 64, 127):
        q = np.tile(np.eye(1, dim), (T, heads, 1)) * 8
        k = np.tile(np.eye(1, dim, 1), (T, kv, 1))
        k[far] = np.eye(1, dim)               # q . k = dim there, 0 elsewhere after the norms
        v = 0.1 * rng.standard_normal((T, kv, vdim))
        v[far] = 1.0
        proj, pv = dev.act(np.concatenate([x.reshape(T, -1) for x in (q, k, v)], axis=1), f32)
        vv = pv[:, (heads + kv) * dim:].reshape(T, kv, vdim)
        want = plain.window_attention(plain.rms(q, 1e-6), plain.rms(k, 1e-6), vv, window, 3.0)
        assert far + window >= T or (want[far + window - 1].min() > 0.9 and want[far + window].max() < 0.5)
        for sizes in ([T], [1], [37, 2, 1, 1], [128, 1]):
            slots = (window - 1 + max(sizes) + 63) // 64 * 64
            got = attend(awq, lib, dev, f32, proj, heads, kv, dim, vdim, window, 3.0, 1e-6, (0.0, 1.0), sizes, T, slots, T)
            assert np.abs(got - want).max() < (1e-4 if f32 else 0.01), (far, sizes)


@pytest.mark.parametrize("f32", FORMATS, ids=["bf16", "f32"])
def test_a_far_key_among_many_and_the_bias(awq, lib, dev, f32):
    """no window: a single key hundreds of positions back carries the answer although the distance bias pulls it down"""
    heads, kv, dim, vdim, T = 8, 4, 128, 64, 700
    q = np.tile(np.eye(1, dim), (T, heads, 1)) * 5
    k = np.tile(np.eye(1, dim, 1), (T, kv, 1))
    v = np.zeros((T, kv, vdim))
    for i, at in enumerate((3, 64, 191, 400)):
        k[at, i] = np.eye(1, dim)
        v[at, i] = 1 + i
    proj, pv = dev.act(np.concatenate([x.reshape(T, -1) for x in (q, k, v)], axis=1), f32)
    want = plain.window_attention(plain.rms(q, 1e-6), plain.rms(k, 1e-6), v, None, 0.3, (0.5, 100))
    assert want[-1].max() > 0.5 and want[-1].min() < 0.01   # heads differ: the bias decides
    for sizes in ([T], [650, 1], [127, 2]):
        got = attend(awq, lib, dev, f32, proj, heads, kv, dim, vdim, 0, 0.3, 1e-6, (0.5, 100.0), sizes, T, 704, T)
        assert np.abs(got - want).max() < (2e-3 if f32 else 0.04), sizes
