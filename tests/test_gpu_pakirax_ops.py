"""The operators of the dense models against plain float64 restatements, both context types: matrix products in every
row class, norms over the residual, gated linear attention in both forms, latent attention in both forms with keys that
stand out at chosen distances."""
import math

import numpy as np
import pytest
import torch

import pakirax_oracle as P
from gpu_util import say

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module", params=["bf16", "fp32"])
def ctx(request):
    import nvmai_amd as nv
    return nv.Context(0, nv.ACT_BF16 if request.param == "bf16" else nv.ACT_FP32)


def is32(ctx):
    return ctx.dtype == torch.float32


def bf(rng, *shape, std=1.0):
    """BF16 values as (device tensor, float64 array)."""
    t = torch.from_numpy((rng.standard_normal(shape) * std).astype(np.float32)).to(torch.bfloat16)
    return t.cuda(), t.double().numpy()


def acts(ctx, a, cols=None):
    """Activations with `cols` columns (zeros past a's own): (device tensor, float64 array of what it holds)."""
    t = torch.zeros((a.shape[0], cols or a.shape[1]), dtype=ctx.dtype)
    t[:, :a.shape[1]] = torch.from_numpy(np.asarray(a, np.float32)).to(ctx.dtype)
    return t.cuda(), t[:, :a.shape[1]].double().numpy()


def close(got, want, tol):
    got = got.double().cpu().numpy() if torch.is_tensor(got) else got
    err = np.abs(got - want).max() / max(1e-30, np.abs(want).max())
    assert err < tol, "max error %.3g of the largest value, allowed %.3g" % (err, tol)


# ---- matrix products ---------------------------------------------------------------------------------
@pytest.mark.parametrize("rows", [1, 2, 3, 4, 5, 16, 17, 33, 64, 65, 130, 300])
@pytest.mark.parametrize("n,k", [(1, 64), (37, 192), (256, 576), (3100, 128), (8197, 64)])
def test_dense_linear(ctx, rows, n, k):
    import nvmai_amd as nv
    say("dense_linear", ctx.dtype, rows, n, k)
    rng = np.random.default_rng(rows * 1000 + n + k)
    w, w64 = bf(rng, n, k, std=k ** -0.5)
    x, x64 = acts(ctx, rng.standard_normal((rows, k)), k + 64)
    want = x64 @ w64.T
    stride = n + 3 if n % 2 else n + 4
    y = torch.full((rows, stride), 7.0, dtype=ctx.dtype, device="cuda")
    y32 = torch.full((rows, stride), 7.0, dtype=torch.float32, device="cuda")
    nv.dense_linear(ctx, w, x, y=y, y_f32=y32)
    close(y32[:, :n], want, 2e-6)
    close(y[:, :n], want, 2e-6 if is32(ctx) else 6e-3)
    assert bool((y[:, n:] == 7).all()) and bool((y32[:, n:] == 7).all())       # nothing beside the outputs
    nv.dense_linear(ctx, w, x, y_f32=y32, activation=nv.LINEAR_GELU_ERF)
    close(y32[:, :n], P.gelu_erf(want), 3e-6)


def test_dense_linear_tiles_cover_large_products():
    import nvmai_amd as nv
    ctx = nv.Context(0, nv.ACT_BF16)
    for rows, n, k in [(1030, 4100, 256), (4096, 520, 128), (700, 2050, 192)]:      # the three tile shapes, ragged edges
        say("dense_linear tiles", rows, n, k)
        rng = np.random.default_rng(n)
        w, w64 = bf(rng, n, k, std=k ** -0.5)
        x, x64 = acts(ctx, rng.standard_normal((rows, k)))
        y = torch.empty((rows, n), dtype=torch.float32, device="cuda")
        nv.dense_linear(ctx, w, x, y_f32=y)
        close(y, x64 @ w64.T, 2e-6)


def test_dense_linear_refuses_what_it_does_not_take():
    import nvmai_amd as nv
    ctx, half = nv.Context(0, nv.ACT_BF16), nv.Context(0, nv.ACT_FP16)
    w = torch.zeros((16, 128), dtype=torch.bfloat16, device="cuda")
    y = torch.zeros((2, 16), dtype=torch.float32, device="cuda")
    with pytest.raises(nv.NvmaiError):
        nv.dense_linear(ctx, w[:, :96].contiguous(), torch.zeros((2, 96), dtype=torch.bfloat16, device="cuda"), y_f32=y)
    with pytest.raises(nv.NvmaiError):
        nv.dense_linear(half, w, torch.zeros((2, 128), dtype=torch.float16, device="cuda"), y_f32=y)
    with pytest.raises(nv.NvmaiError):
        nv.RMSNorm(nv.Context(0, nv.ACT_FP32)).encode_no_scale(torch.zeros((2, 64), device="cuda"))


# ---- norms, rows, argmax -------------------------------------------------------------------------------
@pytest.mark.parametrize("d", [1, 7, 64, 250, 600, 2048, 5000])
def test_norm_residual(ctx, d):
    import nvmai_amd as nv
    say("norm_residual", ctx.dtype, d)
    rng = np.random.default_rng(d)
    rows, eps, mult = 5, 1e-3, 0.37
    (pw, pw64), (pb, pb64), (nw, nw64), (nb, nb64) = (bf(rng, d) for _ in range(4))
    x32, d32 = (rng.standard_normal((rows, d)).astype(np.float32) * 3 + 1 for _ in range(2))
    delta = torch.zeros((rows, d + 5), device="cuda")
    delta[:, :d] = torch.from_numpy(d32)
    for with_delta, with_post in [(True, True), (True, False), (False, False)]:
        x = torch.from_numpy(x32).cuda()
        out = torch.full((rows, d + 3), 9.0, dtype=ctx.dtype, device="cuda")
        nv.norm_residual(ctx, x, d, delta if with_delta else None, (pw, pb) if with_post else None, mult, (nw, nb), out, eps)
        want = x32.astype(np.float64)
        if with_delta:
            want = want + mult * (P.layer_norm(d32.astype(np.float64), pw64, pb64, eps) if with_post else d32)
        close(x, want, 1e-6)
        close(out[:, :d], P.layer_norm(want, nw64, nb64, eps), 3e-6 if is32(ctx) else 5e-3)
        assert bool((out[:, d:] == 9).all())


def test_embed_rows_and_argmax(ctx):
    import nvmai_amd as nv
    rng = np.random.default_rng(3)
    table, t64 = bf(rng, 50, 128)
    ids = torch.tensor([0, 49, 7, 50, 7], dtype=torch.int32, device="cuda")
    out = nv.embed_rows(ctx, table, ids, 100, 50, torch.empty((5, 100), device="cuda"))
    want = np.stack([t64[i, :100] if i < 50 else np.zeros(100) for i in [0, 49, 7, 50, 7]])
    assert np.array_equal(out.double().cpu().numpy(), want)
    x = rng.standard_normal((6, 5003)).astype(np.float32)
    x[1, [17, 4000]] = 9.0          # a tie: the lower index
    x[2, 5002] = 9.0
    x[3, :] = -np.inf
    x[3, 4321] = -5.0
    x[4, 3], x[4, 100] = np.inf, 8.0   # not finite: passed over
    x[5, :] = np.nan
    got = nv.argmax_rows(ctx, torch.from_numpy(x).cuda()).tolist()
    assert got == [int(x[0].argmax()), 17, 5002, 4321, 100, 0]


# ---- gated linear attention -----------------------------------------------------------------------------
def gla_case(ctx, rng, heads, dk, dv, rank, rows, tau, bias, count=None):
    """Device operands of one call and the float64 pieces behind them; `count` = (key, value) counts below the sizes."""
    kc, vc = count or (dk, dv)
    part = lambda n, c: np.where(np.arange(n) % (n // heads) < c, rng.standard_normal((rows, n)), 0.0)
    q, k, v, g = part(heads * dk, kc), part(heads * dk, kc), part(heads * dv, vc), rng.standard_normal((rows, heads * dv))
    a1 = rng.standard_normal((rows, rank))
    proj = torch.from_numpy(np.concatenate([q, k, v, g, a1], 1).astype(np.float32)).cuda()
    p64 = proj.double().cpu().numpy()
    cuts = np.cumsum([0, heads * dk, heads * dk, heads * dv, heads * dv, rank])
    dev = [proj[:, a:] for a in cuts[:5]]
    f64 = [p64[:, a:b] for a, b in zip(cuts, cuts[1:])]
    a2, a2_64 = bf(rng, heads * dk, rank, std=rank ** -0.5)
    b = torch.from_numpy(np.asarray(bias(heads * dk), np.float32)).to(torch.bfloat16)
    nw, nw64 = bf(rng, dv)
    return dev, f64, (a2, b.cuda(), nw), (a2_64, b.double().numpy(), nw64)


def gla_plain(f64, w64, heads, dk, dv, tau, eps, S, count=None):
    kc, vc = count or (dk, dv)
    q, k, v, g, a1 = f64
    a2, b, nw = w64
    out = []
    for t in range(len(q)):
        alpha = P.decay(a2 @ a1[t] + b, tau).reshape(heads, dk)
        rows = []
        for h in range(heads):
            S[h] = alpha[h][:, None] * S[h] + np.outer(k[t].reshape(heads, dk)[h], v[t].reshape(heads, dv)[h])
            o = S[h].T @ (q[t].reshape(heads, dk)[h] * kc ** -0.5)
            o = o / np.sqrt((o[:vc] ** 2).mean() + eps)
            rows.append(o * nw)
        out.append(np.concatenate(rows) * P.silu(g[t]))
    return np.stack(out)


BIASES = {"slow": lambda n: np.full(n, 6.0), "mixed": lambda n: np.linspace(-4, 8, n), "harsh": lambda n: np.where(np.arange(n) % 3, 3.0, -70.0)}


@pytest.mark.parametrize("form", ["recurrent", "chunked"])
@pytest.mark.parametrize("bias", sorted(BIASES))
@pytest.mark.parametrize("heads,dk,dv,rank,rows", [(2, 16, 16, 8, 1), (3, 48, 80, 16, 37), (1, 128, 128, 24, 130), (2, 32, 256, 8, 64),
                                                   (1, 208, 16, 16, 17), (5, 64, 48, 16, 257)])
def test_gla_forms(ctx, form, bias, heads, dk, dv, rank, rows):
    import nvmai_amd as nv
    say("gla", ctx.dtype, form, bias, heads, dk, dv, rank, rows)
    rng = np.random.default_rng(heads + dk * 3 + rows)
    tau, eps = 2.0 if bias != "harsh" else 1.0, 1e-5
    dev, f64, w, w64 = gla_case(ctx, rng, heads, dk, dv, rank, rows, tau, BIASES[bias])
    op = nv.GLA(ctx, heads, dk, dv, rank, tau, eps)
    state = op.new_state(3)
    S = rng.standard_normal((heads, dk, dv)).astype(np.float32)
    state[1] = torch.from_numpy(S)
    out = torch.full((rows, heads * dv + 16), 5.0, dtype=ctx.dtype, device="cuda")
    op.encode(*dev, *w, state, out, rows, slot=1, form=nv.GLA_RECURRENT if form == "recurrent" else nv.GLA_CHUNKED)
    S64 = S.astype(np.float64)
    want = gla_plain(f64, w64, heads, dk, dv, tau, eps, S64)
    close(state[1], S64, 2e-5)
    close(out[:, :heads * dv], want, 3e-5 if is32(ctx) else 6e-3)
    assert bool((state[0] == 0).all()) and bool((state[2] == 0).all()) and bool((out[:, heads * dv:] == 5).all())


def test_gla_counts_below_the_padded_sizes(ctx):
    """Zero-padded heads: scale and norm follow the real sizes."""
    import nvmai_amd as nv
    rng = np.random.default_rng(8)
    heads, dk, dv, rank, rows, count = 2, 32, 48, 16, 70, (19, 37)
    dev, f64, w, w64 = gla_case(ctx, rng, heads, dk, dv, rank, rows, 4.0, BIASES["mixed"], count)
    for form in (nv.GLA_RECURRENT, nv.GLA_CHUNKED):
        op = nv.GLA(ctx, heads, dk, dv, rank, 4.0, 1e-4, *count)
        out = torch.zeros((rows, heads * dv), dtype=ctx.dtype, device="cuda")
        op.encode(*dev, *w, op.new_state(1), out, rows, form=form)
        close(out, gla_plain(f64, w64, heads, dk, dv, 4.0, 1e-4, np.zeros((heads, dk, dv)), count), 3e-5 if is32(ctx) else 6e-3)


def test_gla_batch_of_slots_equals_each_alone(ctx):
    import nvmai_amd as nv
    rng = np.random.default_rng(9)
    heads, dk, dv, rank, B = 3, 48, 32, 8, 5
    dev, _, w, _ = gla_case(ctx, rng, heads, dk, dv, rank, B, 8.0, BIASES["mixed"])
    op = nv.GLA(ctx, heads, dk, dv, rank, 8.0, 1e-5)
    first = torch.randn((7, heads, dk, dv), device="cuda", generator=torch.Generator("cuda").manual_seed(1))
    slots = torch.tensor([6, 0, 3, 2, 5], dtype=torch.int32, device="cuda")
    state, out = first.clone(), torch.zeros((B, heads * dv), dtype=ctx.dtype, device="cuda")
    op.encode(*dev, *w, state, out, 1, B, slots=slots)
    for r, s in enumerate(slots.tolist()):
        alone, o = first.clone(), torch.zeros((1, heads * dv), dtype=ctx.dtype, device="cuda")
        op.encode(*[t[r:r + 1] for t in dev], *w, alone, o, 1, slot=s)
        assert torch.equal(o[0], out[r]) and torch.equal(alone[s], state[s])
    assert torch.equal(state[1], first[1]) and torch.equal(state[4], first[4])


# ---- latent attention -----------------------------------------------------------------------------------
class Latent:
    """One layer's operands and its plain restatement; rows are fed in portions through the library's two calls."""

    def __init__(self, ctx, rng, heads, nope, rot, vdim, rank, window, n, capacity=None, slots=1, count=None, rotary=None, spikes=(), cache_ctx=None):
        import nvmai_amd as nv
        self.nv, self.ctx, self.n, self.window = nv, ctx, n, window
        self.heads, self.nope, self.rot, self.vdim, self.rank = heads, nope, rot, vdim, rank
        self.count = rank if count is None else count
        self.rotary = rot if rotary is None else rotary
        self.eps, self.scale, self.base = 1e-5, 0.4 * (nope + rot) ** -0.5, 3000.0
        qc = 24
        down = rng.standard_normal((n, qc + rank + rot + heads))
        down[:, qc + self.count:qc + rank] = 0.0
        q = rng.standard_normal((n, heads * (nope + rot)))
        self.uk, self.uk64 = bf(rng, heads * nope, rank, std=self.count ** -0.5)
        self.uv, self.uv64 = bf(rng, heads * vdim, rank, std=self.count ** -0.5)
        self.kvn, self.kvn64 = bf(rng, rank)
        self.qn, self.qn64 = bf(rng, qc)
        self.proj, self.p64 = acts(ctx, down, (down.shape[1] + 7) // 8 * 8)
        for i, j in spikes:                         # query i points at key j: W_uk c_j dominates its scores
            c = P.rms_norm(self.p64[j, qc:qc + self.count], self.kvn64[:self.count], self.eps)
            for h in range(heads):
                key = self.uk64[h * nope:(h + 1) * nope, :self.count] @ c
                q[i, h * (nope + rot):h * (nope + rot) + nope] = key / np.linalg.norm(key) ** 2 * (25.0 / self.scale)
        self.q, self.q64 = acts(ctx, q)
        self.qc = qc
        self.op = nv.LatentAttention(ctx, heads, nope, rot, vdim, rank, self.count, self.scale, window, self.rotary, self.base, self.eps)
        self.cache = nv.LatentCache(cache_ctx or ctx, slots, capacity or n, rank, rot)

    def run(self, portions, form, slot=0, base=0):
        """Feed `portions` (row counts) from position base; the gated outputs of every row."""
        nv, at, out = self.nv, 0, []
        for T in portions:
            rows = nv.row_map(slot, base + at)
            proj, q = self.proj[at:at + T], self.q[at:at + T].clone()
            cq = torch.zeros((T, 64), dtype=self.ctx.dtype, device="cuda")
            self.op.encode_epilogue(proj, 0, self.qc, self.qn, self.qc, self.qc + self.rank, self.kvn, cq, self.cache, rows)
            close(cq[:, :self.qc], P.rms_norm(self.p64[at:at + T, :self.qc], self.qn64, self.eps), 1e-6 if is32(self.ctx) else 5e-3)
            y = torch.full((T, self.heads * self.vdim + 4), 3.0, dtype=self.ctx.dtype, device="cuda")
            gate = proj[:, self.qc + self.rank + self.rot:]
            self.op.encode(q, gate, self.uk, self.uv, self.cache, rows, y, form)
            assert bool((y[:, self.heads * self.vdim:] == 3).all())
            out.append(y[:, :self.heads * self.vdim].double().cpu().numpy())
            at += T
        return np.concatenate(out)

    def plain(self, rows, base=0):
        """Expected outputs of `rows` (all of the sequence's rows before them are its keys)."""
        qc, cnt = self.qc, self.count
        c = P.rms_norm(self.p64[:, qc:qc + cnt], self.kvn64[:cnt], self.eps)
        kr = np.stack([P.rotate_half(self.p64[j, qc + self.rank:qc + self.rank + self.rot], base + j, self.base, self.rotary) for j in range(self.n)])
        gate = P.sigmoid(self.p64[:, qc + self.rank + self.rot:])
        out = []
        for i in rows:
            qs = self.q64[i].reshape(self.heads, -1)
            lo = 0 if self.window == 0 else max(0, i - self.window + 1)
            row = []
            for h in range(self.heads):
                k = c[lo:i + 1] @ self.uk64[h * self.nope:(h + 1) * self.nope, :cnt].T
                v = c[lo:i + 1] @ self.uv64[h * self.vdim:(h + 1) * self.vdim, :cnt].T
                s = (k @ qs[h, :self.nope] + kr[lo:i + 1] @ P.rotate_half(qs[h, self.nope:], base + i, self.base, self.rotary)) * self.scale
                w = np.exp(s - s.max())
                row.append(w @ v / w.sum() * gate[i, h])
            out.append(np.concatenate(row))
        return np.stack(out)


def check_latent(ctx, L, got, rows=None, base=0):
    rows = range(L.n) if rows is None else rows
    close(got[list(rows)], L.plain(rows, base), 2e-5 if is32(ctx) else 2e-2)


FORMS = {"absorbed": 1, "expanded": 2}


@pytest.mark.parametrize("form", sorted(FORMS))
@pytest.mark.parametrize("heads,nope,rot,vdim,rank,window,n", [(1, 16, 16, 16, 64, 1, 40), (3, 32, 16, 48, 128, 7, 150), (16, 64, 32, 64, 128, 64, 200),
                                                              (18, 16, 16, 32, 192, 65, 140), (2, 128, 64, 128, 512, 0, 300),
                                                              (2, 48, 32, 160, 320, 100, 270), (1, 208, 48, 256, 576, 30, 70)])
def test_latent_attention_whole_prompt(ctx, form, heads, nope, rot, vdim, rank, window, n):
    say("latent attention", ctx.dtype, form, heads, nope, rot, vdim, rank, window, n)
    rng = np.random.default_rng(heads + n)
    L = Latent(ctx, rng, heads, nope, rot, vdim, rank, window, n)
    check_latent(ctx, L, L.run([n], FORMS[form]))


def test_latent_attention_sizes_past_the_matrix_core_kernels(ctx):
    """Head sizes above 256 and a rank above 1024 take the plain kernels."""
    rng = np.random.default_rng(5)
    L = Latent(ctx, rng, 1, 272, 16, 272, 64, 9, 40)
    check_latent(ctx, L, L.run([40], FORMS["expanded"]))
    L = Latent(ctx, rng, 2, 32, 16, 32, 1088, 9, 40)
    check_latent(ctx, L, L.run([3, 37], FORMS["absorbed"]))
    L = Latent(ctx, rng, 2, 32, 16, 32, 1024, 40, 70)
    check_latent(ctx, L, L.run([3, 67], FORMS["absorbed"]))


@pytest.mark.parametrize("window", [33, 64, 96, 129])
def test_latent_window_edges_in_prompts_and_decoding(ctx, window):
    """Queries that point at one key: just inside the window, just outside it, the first tokens, themselves, far keys
    across tile and split borders."""
    rng = np.random.default_rng(window)
    n = 400
    spikes, used = [], set()
    for d in (0, 1, 31, 32, 63, 64, window - 2, window - 1, window, window + 1):
        for i in (window - 1, window, window + 1, 130 + d, 256, 257, n - 1 - d):
            if 0 <= i - d and i not in used and i < n:
                used.add(i)
                spikes.append((i, i - d))
    L = Latent(ctx, rng, 2, 32, 16, 32, 64, window, n, spikes=spikes)
    rows = sorted(used)
    want = L.plain(rows)
    for name, portions, form in [("prompt", [n], 2), ("prompt, absorbed", [n], 1), ("decoding", [1] * n, 0), ("portions", [2, 61, 64, 33, 5, 100, 135], 0)]:
        say("latent window edges", ctx.dtype, window, name)
        close(L.run(portions, form)[rows], want, 2e-5 if is32(ctx) else 2e-2)
    # the test sees the edge: with a window one token off, the spiked rows differ by far more than that
    L.window = window + 1
    assert np.abs(L.plain(rows) - want).max() > 0.1 * np.abs(want).max()


def test_latent_ring_wraps_and_slots_are_reused(ctx):
    """A ring much shorter than the sequence, portions that end at and straddle its end, a slot used again at once."""
    import nvmai_amd as nv
    rng = np.random.default_rng(21)
    window, n = 40, 333
    L = Latent(ctx, rng, 3, 32, 16, 32, 64, window, n, capacity=40 + 60 - 1, slots=3)
    want = L.plain(range(n))
    for slot, portions in [(1, [60, 39, 1, 59, 60, 2, 58, 54]), (2, [1] * 100 + [60, 3] + [1] * 170), (1, [33, 60, 60, 60, 60, 60])]:
        say("latent ring", ctx.dtype, slot, portions[:6])
        close(L.run(portions, nv.FORM_AUTO, slot=slot), want, 2e-5 if is32(ctx) else 2e-2)
    assert bool((L.cache.rows[0] == 0).all())
    with pytest.raises(nv.NvmaiError):
        L.run([61], nv.FORM_AUTO, base=100)         # window + 60 rows do not fit the ring


def test_latent_positions_far_along_and_partial_rotation(ctx):
    """Large positions (the angle is reduced in double) and a rotation of a part of the rope dims."""
    rng = np.random.default_rng(31)
    for base, rotary in [(100003, 16), (0, 6), (5, 0)]:
        L = Latent(ctx, rng, 2, 16, 16, 16, 64, 20, 50, count=41, rotary=rotary, capacity=128)
        # rows whose window lies inside what was fed (positions before `base` were not)
        rows = list(range(0 if base == 0 else 19, 50))
        for portions in ([50], [1] * 50):
            close(L.run(portions, 0, base=base)[rows], L.plain(rows, base), 2e-5 if is32(ctx) else 2e-2)


def test_latent_decode_batch_of_unequal_positions(ctx):
    import nvmai_amd as nv
    rng = np.random.default_rng(41)
    window, n, B = 50, 230, 4
    Ls = [Latent(ctx, np.random.default_rng(41), 5, 32, 16, 48, 128, window, n, slots=6)]
    L = Ls[0]
    lengths, slots = [1, 50, 51, 229], [5, 0, 3, 2]
    for s, m in zip(slots, lengths):
        L.run([m], 0, slot=s)
    pos = torch.tensor(lengths, dtype=torch.int32, device="cuda")
    sl = torch.tensor(slots, dtype=torch.int32, device="cuda")
    rows = nv.row_map(slots=sl, positions=pos)
    pick = torch.tensor(lengths, device="cuda")
    proj, q = L.proj[pick].contiguous(), L.q[pick].contiguous()
    cq = torch.zeros((B, 64), dtype=ctx.dtype, device="cuda")
    L.op.encode_epilogue(proj, 0, L.qc, L.qn, L.qc, L.qc + L.rank, L.kvn, cq, L.cache, rows)
    y = torch.zeros((B, L.heads * L.vdim), dtype=ctx.dtype, device="cuda")
    L.op.encode(q, proj[:, L.qc + L.rank + L.rot:], L.uk, L.uv, L.cache, rows, y)
    close(y, L.plain(lengths), 2e-5 if is32(ctx) else 2e-2)


def test_latent_attention_in_32_bit_over_a_bf16_cache():
    """32-bit rows beside a BF16 cache: what passes of one or two rows use.  The cached rows and the query on its way to them are
    BF16, everything else 32-bit; the expanded form is refused."""
    import nvmai_amd as nv
    full, half = nv.Context(0, nv.ACT_FP32), nv.Context(0, nv.ACT_BF16)
    for window, portions in [(33, [1] * 90), (64, [4, 3, 2, 1] * 9), (0, [50, 40])]:
        n = sum(portions)
        L = Latent(full, np.random.default_rng(window), 5, 48, 32, 48, 128, window, n, cache_ctx=half)
        close(L.run(portions, nv.FORM_AUTO), L.plain(range(n)), 1e-2)
    with pytest.raises(nv.NvmaiError):
        L.run([90], nv.LATENT_EXPANDED)
    with pytest.raises(nv.NvmaiError):
        Latent(half, np.random.default_rng(0), 5, 48, 32, 48, 128, 33, 4, cache_ctx=full).run([4], nv.FORM_AUTO)
