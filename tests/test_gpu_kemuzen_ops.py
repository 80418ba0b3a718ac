"""Operators behind the Kemuzen model against the plain oracle or float64 restatements: the products' further epilogues,
RMS norms over the residual, embeddings with sinusoids, windowed attention with kept first tokens in its three forms, the
recurrences with one decay per head in both forms, the gated norm.  Sizes off every tile, queries and keys that make
single positions stand out."""
import math

import numpy as np
import pytest
import torch

import kemuzen_oracle as K
from gpu_util import say

pytestmark = pytest.mark.gpu
TYPES = ["bfloat16", "float32"]


def context(dtype):
    import nvmai_amd as nv
    return nv.Context(0, nv.ACT_BF16 if dtype == "bfloat16" else nv.ACT_FP32)


def randn(seed, *shape, std=1.0):
    return torch.from_numpy((np.random.default_rng(seed).standard_normal(shape) * std).astype(np.float32)).cuda()


def bf(t):
    return t.to(torch.bfloat16)


def f64(t):
    return t.double().cpu().numpy()


def close(got, want, bar, what, least=1e-30):
    e = np.abs(got - want).max() / max(least, np.abs(want).max())
    assert e < bar, "%s: off by %.3g of the largest value" % (what, e)


# ---- products -------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", TYPES)
@pytest.mark.parametrize("rows", [1, 2, 3, 4, 5, 17, 40, 64, 70, 300])
def test_products_with_bias_activation_and_multiplier(dtype, rows):
    import nvmai_amd as nv
    ctx = context(dtype)
    n, k, vocab = 52, 192, 30
    w, x, bias = bf(randn(1, n, k, std=k ** -0.5)), randn(2, rows, k).to(ctx.dtype), bf(randn(3, n))
    table = bf(randn(4, vocab, 3 * n + 5))
    ids = torch.from_numpy(np.random.default_rng(5).integers(0, vocab, rows).astype(np.int32)).cuda()
    ids[rows // 2] = vocab + 3                       # past the table: multiplied by zero
    part = table[:, n + 1:2 * n + 1]
    say("dense_linear_ex", dtype, rows)
    base = f64(x) @ f64(w).T
    bar = 2e-6 if dtype == "float32" else 1e-5
    mul = np.where((f64(ids) < vocab)[:, None], f64(part)[np.minimum(ids.cpu().numpy(), vocab - 1)], 0.0)
    for what, kw, want in [("bias", dict(bias=bias), base + f64(bias)),
                           ("gelu", dict(activation=nv.LINEAR_GELU_TANH), K.gelu_tanh(base)),
                           ("all", dict(bias=bias, activation=nv.LINEAR_GELU_TANH, mul=part, mul_ids=ids), K.gelu_tanh(base + f64(bias)) * mul)]:
        y, y32 = torch.zeros((rows, 64), dtype=ctx.dtype, device="cuda"), torch.zeros((rows, 64), device="cuda")
        nv.dense_linear(ctx, w, x, y=y, y_f32=y32, **kw)
        close(f64(y32)[:, :n], want, bar, what)
        assert torch.equal(y32.to(ctx.dtype), y) and not y32[:, n:].any()


@pytest.mark.parametrize("dtype", TYPES)
@pytest.mark.parametrize("rows", [1, 2, 3, 4, 6, 33, 64, 65, 300])
@pytest.mark.parametrize("n", [2, 50, 134, 9000])
def test_products_of_gate_and_up_rows_in_turn(dtype, rows, n):
    import nvmai_amd as nv
    ctx = context(dtype)
    k = 128
    w, x = bf(randn(1, n, k, std=k ** -0.5)), randn(2, rows, k).to(ctx.dtype)
    base = f64(x) @ f64(w).T
    want = K.silu(base[:, 0::2]) * base[:, 1::2]
    say("silu pairs", dtype, rows, n)
    stride = n // 2 + 5 + (n // 2 + 5) % 2
    y, y32 = torch.zeros((rows, stride), dtype=ctx.dtype, device="cuda"), torch.zeros((rows, stride), device="cuda")
    nv.dense_linear(ctx, w, x, y=y, y_f32=y32, activation=nv.LINEAR_SILU_PAIRS)
    close(f64(y32)[:, :n // 2], want, 3e-6 if dtype == "float32" else 2e-5, "pairs", least=1.0)
    assert torch.equal(y32.to(ctx.dtype), y) and not y32[:, n // 2:].any()


# ---- norms, embeddings -------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", TYPES)
@pytest.mark.parametrize("d,stride", [(1, 3), (5, 8), (72, 72), (72, 75), (1024, 1024), (1500, 1500), (2048, 2048), (5000, 5000)])
def test_rms_norms_over_the_residual(dtype, d, stride):
    import nvmai_amd as nv
    ctx, rows, eps = context(dtype), 3, 1e-3
    post, nxt = bf(randn(3, d)), bf(randn(4, d))
    say("rms_residual", dtype, d, stride)
    for add_p, add_n in ((0.0, 1.0), (1.0, 0.0)):
        for kind in ("copy", "norm", "none", "norm only"):
            x, delta = randn(1, rows, stride), randn(2, rows, stride, std=3.0)
            want = f64(x)[:, :d]
            out = torch.full((rows, stride), 7.0, dtype=ctx.dtype, device="cuda")
            only = kind == "norm only"
            nv.rms_residual(ctx, x, d, None if only else delta, None if only else post, add_p, nxt if kind.startswith("norm") else None, add_n,
                            None if kind == "none" else out, eps)
            if not only:
                want = want + K.rms(f64(delta)[:, :d], eps) * (add_p + f64(post))
            close(f64(x)[:, :d], want, 1e-6, "residual")
            if kind != "none":
                o = K.rms(want, eps) * (add_n + f64(nxt)) if kind.startswith("norm") else want
                close(f64(out)[:, :d], o, 2e-6 if dtype == "float32" else 5e-3, kind)
            assert (out[:, d:] == 7.0).all()


@pytest.mark.parametrize("dtype", TYPES)
@pytest.mark.parametrize("width", [1, 5, 72, 700])
def test_embeddings_with_sinusoids(dtype, width):
    import nvmai_amd as nv
    ctx, vocab = context(dtype), 19
    table = bf(randn(1, vocab, width + 3))
    ids = torch.tensor([4, 18, 0, 99, 4], dtype=torch.int32, device="cuda")
    freq = nv.sinusoid_frequencies(width, ctx.device)
    where = [0, 1, 2, 1000003, 7]
    positions, slots = torch.tensor(where, dtype=torch.int32, device="cuda"), torch.zeros(5, dtype=torch.int32, device="cuda")
    e = np.where(f64(ids)[:, None] < vocab, f64(table)[np.minimum(ids.cpu().numpy(), vocab - 1), :width], 0.0) * 2.5
    for rows_at, at in ((nv.row_map(slots=slots, positions=positions), where), (nv.row_map(0, 65530), range(65530, 65535))):
        out, act = torch.zeros((5, width + 2), device="cuda"), torch.zeros((5, width + 4), dtype=ctx.dtype, device="cuda")
        nv.embed_positions(ctx, table, ids, width, vocab, 2.5, freq, rows_at, out, act)
        want = e + np.stack([K.sinusoid(p, width) for p in at])
        close(f64(out)[:, :width], want, 1e-6, "embedding")
        assert torch.equal(act[:, :width], out[:, :width].to(ctx.dtype)) and not act[:, width:].any()
    nv.embed_positions(ctx, table, ids, width, vocab, 2.5, None, nv.row_map(0, 3), out)
    close(f64(out)[:, :width], e, 1e-6, "no sinusoid")


def test_softcap_of_rows():
    import nvmai_amd as nv
    x = randn(1, 3, 301, std=40.0)
    y = x[:, :300].clone()
    nv.softcap_rows(context("float32"), x[:, :300], 9.0)
    close(f64(x)[:, :300], K.softcap(f64(y), 9.0), 1e-6, "softcap")


# ---- windowed attention ---------------------------------------------------------------------------------------
def up(n, m):
    return (n + m - 1) // m * m


class Window:
    """One attention layer whose projections are given: rows [q | k | v | gate] with padded heads, and the same rows
    through the oracle."""

    def __init__(self, dtype, H, G, dim, vdim, size, keep, softcap=0.0, alibi=False, gate=False, scale=None, slots=1, capacity=None, max_rows=512):
        import nvmai_amd as nv
        self.nv, self.ctx = nv, context(dtype)
        self.H, self.G, self.dim, self.vdim = H, G, dim, vdim
        self.dp, self.vp = up(dim, 32), up(vdim, 16)
        self.m = {"heads": H, "kv_heads": G, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5, "softcap": softcap,
                  "mask": {"size": size, "keep_first": keep} if size else None}
        self.alibi, self.gate, self.eps = alibi, gate, 1e-5
        self.op = nv.WindowAttention(self.ctx, H, dim, self.m["scale"], size or 0, self.eps, keep, softcap, alibi)
        self.cache = nv.KvRing(self.ctx, slots, G, self.dp, self.vp, capacity or 1024, keep)
        self.qn, self.kn = bf(1.0 + 0.2 * randn(91, dim)), bf(1.0 + 0.2 * randn(92, dim))
        pad = lambda w: torch.cat([w, torch.zeros(self.dp - dim, dtype=w.dtype, device="cuda")])
        self.qnp, self.knp = pad(self.qn), pad(self.kn)
        self.at = dict(q=0, k=H * self.dp, v=(H + G) * self.dp, g=(H + G) * self.dp + G * self.vp)
        self.cols = self.at["g"] + up(H, 4)

    def rows(self, seed, n, sharp=3.0):
        """Real columns [n, heads, size] of q, k, v and one gate per head."""
        r = np.random.default_rng(seed)
        f = lambda *s: r.standard_normal(s).astype(np.float32)
        return [f(n, self.H, self.dim) * sharp, f(n, self.G, self.dim), f(n, self.G, self.vdim), f(n, self.H)]

    def proj(self, q, k, v, g):
        out = np.zeros((len(q), self.cols), np.float32)
        for name, x, p in (("q", q, self.dp), ("k", k, self.dp), ("v", v, self.vp)):
            for h in range(x.shape[1]):
                out[:, self.at[name] + h * p:self.at[name] + h * p + x.shape[2]] = x[:, h]
        out[:, self.at["g"]:self.at["g"] + self.H] = g
        return torch.from_numpy(out).cuda()

    def run(self, data, rows_at, form=0, keys=True):
        proj, n = self.proj(*data), len(data[0])
        q = torch.zeros((n, self.H * self.dp), dtype=self.cache.k.dtype, device="cuda")
        self.op.encode_epilogue(proj, self.at["q"], self.at["k"], self.at["v"], self.qnp, self.knp if keys else None, q, self.cache, rows_at)
        out = torch.full((n, self.H * self.vp + 4), 9.0, dtype=self.ctx.dtype, device="cuda")
        self.op.encode(q, self.cache, rows_at, out, proj[:, self.at["g"]:] if self.gate else None, 0.75, form)
        assert (out[:, self.H * self.vp:] == 9.0).all()
        o = f64(out)[:, :self.H * self.vp].reshape(n, self.H, self.vp)
        assert not o[:, :, self.vdim:].any()
        return o[:, :, :self.vdim].reshape(n, -1)

    def want(self, data, state=None, start=0, sharp=None):
        q, k, v, g = (x.astype(np.float64) for x in data)
        h = np.concatenate([q.reshape(len(q), -1), k.reshape(len(q), -1), v.reshape(len(q), -1), g], 1)
        eye, cut = np.eye(h.shape[1]), np.cumsum([0, self.H * self.dim, self.G * self.dim, self.G * self.vdim, self.H])
        t = {n: eye[a:b] for n, a, b in zip(("q", "k", "v", "g"), cut[:-1], cut[1:]) if n != "g" or self.gate}
        t.update({"q.norm": f64(self.qn), "k.norm": f64(self.kn)})
        return 0.75 * K.attention_rows(t, self.m, self.eps, h, start, {"k": [], "v": []} if state is None else state, alibi=self.alibi)


def bar(dtype):
    return 3e-6 if dtype == "float32" else 2e-2


SHAPES = [(6, 2, 20, 24), (4, 4, 64, 64), (8, 1, 96, 128), (34, 2, 128, 48), (3, 3, 160, 144), (1, 1, 1, 1)]
MASKS = [(17, 3), (64, 64), (1, 0), (33, 70), (44, 7), (None, 0)]


@pytest.mark.parametrize("dtype", TYPES)
@pytest.mark.parametrize("shape", SHAPES)
def test_window_attention_forms_and_masks(dtype, shape):
    import nvmai_amd as nv
    n = 150
    for j, (size, keep) in enumerate(MASKS):
        for softcap, alibi, gate in ((0.0, False, False), (6.0, False, True), (0.0, True, True), (9.0, True, False))[j % 2::2]:
            w = Window(dtype, *shape, size, keep, softcap, alibi, gate)
            data = w.rows(j, n, 1.0 if shape[2] == 1 else 3.0)
            want = w.want(data)
            for form in (nv.FORM_AUTO, nv.WINDOW_PLAIN) if dtype == "float32" else (nv.WINDOW_FLASH, nv.WINDOW_SPLIT, nv.WINDOW_PLAIN):
                say("window", dtype, shape, size, keep, softcap, alibi, form)
                close(w.run(data, nv.row_map(0, 0), form), want, bar(dtype), "form %d mask %s" % (form, (size, keep)))


@pytest.mark.parametrize("softcap", [2.0, 30.0, 50.0, 70.0])
def test_window_attention_under_a_cap_with_scores_at_both_ends(softcap):
    """Scores far past the cap on either side, and rows that see nothing but the lowest ones."""
    import nvmai_amd as nv
    w = Window("bfloat16", 4, 2, 64, 64, 48, 5, softcap, scale=1.0)
    data = w.rows(4, 200)
    data[0][50:60] = 40.0                            # queries and keys along one direction: after the norms q . k = +- 64 and more
    data[1][:100] = -1.0
    data[1][100:] += 0.5
    want = w.want(data)
    for form in (nv.WINDOW_FLASH, nv.WINDOW_SPLIT, nv.WINDOW_PLAIN):
        say("window cap", softcap, form)
        close(w.run(data, nv.row_map(0, 0), form), want, bar("bfloat16"), "form %d" % form)


@pytest.mark.parametrize("dtype", TYPES)
@pytest.mark.parametrize("size,keep", [(17, 3), (44, 7), (5, 70), (64, 0), (31, 33)])
def test_window_ring_wraps_and_kept_tokens_stay(dtype, size, keep):
    """Portions of unequal sizes through a ring just large enough, in both slots of a cache, then tokens one by one in a batch."""
    import nvmai_amd as nv
    portions = [1, 2, 33, 64, 3, 50, 2, 7, 64, 64, 31, 16]
    w = Window(dtype, 4, 2, 32, 32, size, keep, 8.0, slots=2, capacity=size + 63)
    n = sum(portions)
    data = [w.rows(s, n + 20) for s in (1, 2)]
    want = [w.want(d) for d in data]
    at = 0
    for count in portions:
        for slot in (1, 0):
            say("window ring", dtype, size, keep, at, count, slot)
            got = w.run([x[at:at + count] for x in data[slot]], nv.row_map(slot, at))
            close(got, want[slot][at:at + count], bar(dtype), "rows %d + %d" % (at, count))
        at += count
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device="cuda")
    for t in range(at, at + 20):
        pair = [np.stack([data[1][k][t], data[0][k][t - 1 if t > at else t]]) for k in range(4)]
        where = [t, t - 1 if t > at else t]          # the second sequence is one token behind (its first one comes twice)
        got = w.run(pair, nv.row_map(slots=i32([1, 0]), positions=i32(where), most=t))
        close(got, np.stack([want[1][where[0]], want[0][where[1]]]), bar(dtype), "token %d" % t)


@pytest.mark.parametrize("dtype", TYPES)
@pytest.mark.parametrize("size,keep", [(44, 7), (64, 3), (127, 1), (300, 65)])
def test_single_keys_at_the_edges_of_a_window(dtype, size, keep):
    """One key that outweighs all others, put just inside and just outside the window and the kept tokens: its value shows
    or does not."""
    import nvmai_amd as nv
    w = Window(dtype, 2, 1, 32, 32, size, keep, 0.0, capacity=1024, scale=1.0)
    n, q_at = 420, 400
    data = w.rows(3, n, 0.05)
    i = q_at
    for j in (i, i - 1, i - size + 1, i - size, i - size - 1, keep - 1, keep, keep + 1, 0, 64, 127, 128):
        if not 0 <= j <= i:
            continue
        d = [x.copy() for x in data]
        d[0][i] = 1.0                                # after the norms: a score of 32 against about 0
        d[1][:, 0] -= d[1][:, 0].mean(-1, keepdims=True)
        d[1][j] = 1.0
        d[2][j] = 50.0
        want = w.want([x[:i + 1] for x in d])[i]
        seen = i - j < size or j < keep
        assert (want > 30.0 * 0.75).all() == seen
        say("window edge", dtype, size, keep, j)
        for form in (nv.WINDOW_PLAIN,) if dtype == "float32" else (nv.WINDOW_FLASH, nv.WINDOW_SPLIT):
            close(w.run(d, nv.row_map(0, 0), form)[i], want, bar(dtype), "key %d" % j)
        w.run([x[:i] for x in d], nv.row_map(0, 0))
        close(w.run([x[i:i + 1] for x in d], nv.row_map(0, i))[0], want, bar(dtype), "key %d, decoded" % j)


def test_a_layer_uses_another_layers_cache():
    import nvmai_amd as nv
    for dtype in TYPES:
        a, b = Window(dtype, 4, 2, 32, 48, 17, 3, 8.0), Window(dtype, 4, 2, 32, 48, 60, 40, 5.0)
        b.cache = nv.KvRing(a.ctx, 1, 2, 32, 48, 60 + 63, 40)
        a.cache = b.cache
        da, db = a.rows(1, 200), b.rows(2, 200)
        state = {"k": [], "v": []}
        wa = a.want(da, state)
        db = [db[0], da[1], da[2], db[3]]
        wb = b.want(db)
        for lo, hi in ((0, 64), (64, 66), (66, 67), (67, 130), (130, 194), (194, 200)):
            say("shared cache", dtype, lo)
            close(a.run([x[lo:hi] for x in da], nv.row_map(0, lo)), wa[lo:hi], bar(dtype), "owner")
            close(b.run([x[lo:hi] for x in db], nv.row_map(0, lo), keys=False), wb[lo:hi], bar(dtype), "user")


def test_few_rows_in_32_bits_over_a_bf16_cache():
    import nvmai_amd as nv
    w = Window("bfloat16", 8, 2, 96, 80, 44, 7, 8.0, gate=True)
    data = w.rows(1, 130)
    want = w.want(data)
    w.run([x[:128] for x in data], nv.row_map(0, 0))
    few = nv.Context(0, nv.ACT_FP32)
    w.ctx, w.op = few, nv.WindowAttention(few, 8, 96, w.m["scale"], 44, w.eps, 7, 8.0)
    for form in (nv.WINDOW_SPLIT, nv.WINDOW_PLAIN):
        close(w.run([x[128:] for x in data], nv.row_map(0, 128), form), want[128:], 1e-2, "two rows")


def test_window_attention_refuses_what_does_not_fit():
    import nvmai_amd as nv
    w = Window("bfloat16", 4, 2, 32, 32, 44, 7, capacity=64)
    with pytest.raises(nv.NvmaiError):
        w.run(w.rows(1, 64), nv.row_map(0, 64))      # 44 + 63 positions in a ring of 64
    with pytest.raises(nv.NvmaiError):
        nv.WindowAttention(w.ctx, 3, 32, 1.0, 44, 1e-5, 7).encode_epilogue(torch.zeros((1, w.cols), device="cuda"), 0, 0, 0, w.qnp, w.knp,
                                                                             torch.zeros((1, 96), dtype=torch.bfloat16, device="cuda"), w.cache, nv.row_map(0, 0))


# ---- recurrences --------------------------------------------------------------------------------------------------
class Scan:
    def __init__(self, kind, H, G, dk, dv, taps, slots=1, bias=True, decay=(-2.0, 2.0)):
        import nvmai_amd as nv
        self.nv, self.ctx, self.kind = nv, context("float32"), kind
        self.H, self.G, self.dk, self.dv, self.taps = H, G, dk, dv, taps
        self.kp, self.vp = up(dk, 16), up(dv, 16)
        self.channels = 2 * G * self.kp + H * self.vp
        self.a_at, self.b_at = self.channels, self.channels + H
        self.cols = self.channels + 2 * H + 3
        self.delta = kind == nv.SCAN_DELTA
        self.op = nv.HeadScan(self.ctx, kind, H, G, self.kp, self.vp, taps, 0, self.a_at, self.b_at, dk ** -0.5 if self.delta else 1.0)
        r = np.random.default_rng(7)
        conv = r.standard_normal((2 * G * dk + H * dv, taps)) * 0.5
        conv[:, -1] += 0.6
        cb = r.standard_normal(2 * G * dk + H * dv) * 0.3 if bias else None
        self.conv, self.bias = bf(torch.from_numpy(conv).cuda()), None if cb is None else bf(torch.from_numpy(cb).cuda())
        self.a_log = bf(torch.from_numpy(r.uniform(*decay, H)).cuda())
        self.dt_bias, self.skip = bf(randn(8, H)), bf(randn(9, H))
        self.real = np.concatenate([np.arange(dk) + g * self.kp for g in range(2 * G)] + [2 * G * self.kp + np.arange(dv) + h * self.vp for h in range(H)])
        pad = lambda x: torch.zeros((self.channels,) + x.shape[1:], dtype=x.dtype, device="cuda").index_copy_(0, torch.from_numpy(self.real).cuda(), x)
        self.conv_p, self.bias_p = pad(self.conv), None if cb is None else pad(self.bias)
        self.history, self.state = self.op.new_state(slots)

    def rows(self, seed, n):
        return np.random.default_rng(seed).standard_normal((n, len(self.real) + 2 * self.H)).astype(np.float32)

    def run(self, rows, rows_at, form=0):
        proj = np.zeros((len(rows), self.cols), np.float32)
        c = len(self.real)
        proj[:, self.real] = rows[:, :c]
        proj[:, self.a_at:self.a_at + 2 * self.H] = rows[:, c:]
        by_heads = len(rows) % 2 == 0                # the output head by head or row by row
        out = torch.full((len(rows), self.H * self.vp + 4), 9.0, device="cuda")
        view = out.flatten()[:len(rows) * self.H * self.vp].view(self.H, len(rows), self.vp) if by_heads else \
            out[:, :self.H * self.vp].unflatten(1, (self.H, self.vp)).transpose(0, 1)
        self.op.encode(torch.from_numpy(proj).cuda(), self.conv_p, self.bias_p, self.a_log, self.dt_bias, self.skip, self.history, self.state,
                       rows_at, view, form)
        assert (out.flatten()[len(rows) * self.H * self.vp:] if by_heads else out[:, self.H * self.vp:] == 9.0).all()
        o = f64(view).transpose(1, 0, 2)
        assert not o[:, :, self.dv:].any()
        return o[:, :, :self.dv]

    def want(self, rows):
        H, G, dk, dv, c = self.H, self.G, self.dk, self.dv, len(self.real)
        S, past, out = np.zeros((H, dk, dv)), [], np.zeros((len(rows), H, dv))
        rate, dt_bias, skip = np.exp(f64(self.a_log)), f64(self.dt_bias), f64(self.skip)
        for t, row in enumerate(rows.astype(np.float64)):
            z = K.short_conv(past, row[:c], f64(self.conv), None if self.bias is None else f64(self.bias))
            q, k, v = z[:G * dk].reshape(G, dk), z[G * dk:2 * G * dk].reshape(G, dk), z[2 * G * dk:].reshape(H, dv)
            step = K.softplus(row[c:c + H] + dt_bias)
            for h in range(H):
                j = h // (H // G)
                if self.delta:
                    S[h], out[t, h] = K.delta_step(S[h], K.unit(q[j]) * dk ** -0.5, K.unit(k[j]), v[h], K.sigmoid(row[c + H + h]), np.exp(-rate[h] * step[h]))
                else:
                    S[h], out[t, h] = K.ssd_step(S[h], v[h], k[j], q[j], step[h], rate[h], skip[h])
        self.last = S
        return out

    def state_error(self, slot):
        got = f64(self.state)[slot][:, :self.dk, :self.dv]
        return np.abs(got - self.last).max() / np.abs(self.last).max()


SCANS = [(4, 2, 24, 40, 3), (3, 3, 64, 16, 4), (2, 1, 128, 128, 4), (2, 2, 160, 48, 1), (1, 1, 1, 1, 2), (6, 1, 16, 20, 7), (1, 1, 256, 80, 4)]


@pytest.mark.parametrize("kind", [0, 1])
@pytest.mark.parametrize("shape", SCANS)
def test_scan_forms_match_the_oracle(kind, shape):
    """The recurrent and the chunked form over a whole prompt, lengths on and off the chunk of 64."""
    import nvmai_amd as nv
    for n in (1, 63, 64, 65, 150):
        s = Scan(kind, *shape, slots=2, bias=kind == 1)
        rows = s.rows(n, n)
        want = s.want(rows)
        for slot, form in ((0, nv.SCAN_RECURRENT), (1, nv.SCAN_CHUNKED)):
            say("scan", kind, shape, n, form)
            close(s.run(rows, nv.row_map(slot, 0), form), want, 5e-6, "form %d, %d rows" % (form, n))
            assert s.state_error(slot) < 5e-6


@pytest.mark.parametrize("kind", [0, 1])
@pytest.mark.parametrize("taps", [1, 4, 6])
def test_scan_portions_carry_state_and_filter_inputs(kind, taps):
    import nvmai_amd as nv
    s = Scan(kind, 4, 2, 32, 48, taps, slots=3)
    portions = [2, 1, 3, 64, 33, 1, 1, 5, 31, 32, 130, 2, 40]
    n = sum(portions)
    rows = [s.rows(11 + k, n + 12) for k in range(2)]
    want = [s.want(r) for r in rows]
    at = 0
    for count in portions:
        for seq, slot in ((0, 2), (1, 0)):
            say("scan portions", kind, taps, at, count)
            close(s.run(rows[seq][at:at + count], nv.row_map(slot, at)), want[seq][at:at + count], 1e-5, "rows %d + %d" % (at, count))
        at += count
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device="cuda")
    for t in range(at, at + 12):                     # one token of both, in a batch
        got = s.run(np.stack([rows[1][t], rows[0][t]]), nv.row_map(slots=i32([0, 2]), positions=i32([t, t])))
        close(got, np.stack([want[1][t], want[0][t]]), 1e-5, "token %d" % t)
    s.state[2].zero_()                               # the slot again, from the start: what the filter saw before is not read
    again = s.rows(30, 70)
    close(s.run(again[:3], nv.row_map(2, 0)), s.want(again)[:3], 1e-5, "slot used again")
    close(s.run(again[3:], nv.row_map(2, 3)), s.want(again)[3:], 1e-5, "slot used again, prompt")


@pytest.mark.parametrize("kind", [0, 1])
def test_scan_with_decays_from_none_to_total(kind):
    """Heads that keep everything and heads that forget everything at single tokens, in one chunk: the decay between two
    late rows is exact behind a row that has forgotten all."""
    import nvmai_amd as nv
    s = Scan(kind, 4, 4, 32, 32, 4, slots=2, decay=(-6.0, 5.0))
    rows = s.rows(5, 200)
    c = len(s.real)
    rows[:, c:c + 4] = -6.0
    rows[20::37, c:c + 4] = 60.0
    want = s.want(rows)
    for slot, form in ((0, nv.SCAN_RECURRENT), (1, nv.SCAN_CHUNKED)):
        close(s.run(rows, nv.row_map(slot, 0), form), want, 1e-5, "form %d" % form)
        assert s.state_error(slot) < 1e-5


@pytest.mark.parametrize("kind", [0, 1])
@pytest.mark.parametrize("shape,n", [((16, 8, 128, 128, 4), 12), ((32, 2, 40, 64, 3), 9), ((2, 2, 16, 32, 4), 3)])
def test_scan_of_a_batch(kind, shape, n):
    """One token of many sequences at different places, small and large launches."""
    import nvmai_amd as nv
    s = Scan(kind, *shape, slots=n + 1)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device="cuda")
    starts = [1 + 5 * j % 37 for j in range(n)]
    rows = [s.rows(40 + j, starts[j] + 3) for j in range(n)]
    want = [s.want(r) for r in rows]
    for j in range(n):
        s.run(rows[j][:starts[j]], nv.row_map(n - j, 0))
    for t in range(3):
        say("scan batch", kind, shape, t)
        got = s.run(np.stack([rows[j][starts[j] + t] for j in range(n)]),
                    nv.row_map(slots=i32([n - j for j in range(n)]), positions=i32([x + t for x in starts])))
        close(got, np.stack([want[j][starts[j] + t] for j in range(n)]), 1e-5, "token %d" % t)


@pytest.mark.parametrize("dtype", TYPES)
@pytest.mark.parametrize("heads,dv,parts", [(1, 4096, 1), (9, 512, 1), (3, 128, 3), (2, 256, 2), (4, 40, 4), (6, 20, 4), (6, 20, 1), (3, 16, 3), (64, 64, 2), (40, 72, 1), (1, 1, 1), (1, 700, 1)])
def test_gated_norm(dtype, heads, dv, parts):
    import nvmai_amd as nv
    ctx, rows, vp = context(dtype), 5, up(dv, 16)
    x, z = randn(1, rows, heads, vp), randn(2, rows, heads, vp, std=2.0)
    x[:, :, dv:] = 0.0
    xr, zr = f64(x)[:, :, :dv].reshape(rows, -1), f64(z)[:, :, :dv].reshape(rows, -1)
    for first in (True, False):
        w = bf(randn(3, heads, vp)) if first else bf(randn(3, vp))
        wr = f64(w)[:, :dv].reshape(-1) if first else np.tile(f64(w)[:dv], heads)
        say("gated_norm", dtype, heads, dv, parts, first)
        out = torch.full((rows, heads * vp + 8), 9.0, dtype=ctx.dtype, device="cuda")
        by_heads = x.transpose(0, 1).contiguous() if first else x.transpose(0, 1)
        nv.gated_norm(ctx, by_heads, z.reshape(rows, -1), w, out, dv, parts, first, 1e-5, 1.5)
        n = xr * K.silu(zr) if first else xr
        n = K.rms(n.reshape(rows, parts, -1), 1e-5).reshape(rows, -1) * wr * 1.5
        want = n if first else n * K.silu(zr)
        got = f64(out)[:, :heads * vp].reshape(rows, heads, vp)
        close(got[:, :, :dv].reshape(rows, -1), want, 3e-6 if dtype == "float32" else 5e-3, "gated norm")
        assert (got[:, :, dv:] == 9.0).all() and (out[:, heads * vp:] == 9.0).all()
