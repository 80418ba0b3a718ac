"""Host side of the Kemuzen model (no GPU): configuration, registry, weight layout, and the oracle's own identities."""
import json

import numpy as np
import pytest
import torch

import kemuzen_models as M
import kemuzen_oracle as K
from pakirax_models import logit_error, numpy64, tokens, write_model


def copy(c):
    return json.loads(json.dumps(c))


# ---- configuration and registry ---------------------------------------------------------------------
def test_config_reads_every_layer_by_itself():
    from nvmai_amd.kemuzen import KemuzenConfig
    c = KemuzenConfig(M.MODELS["mixed"])
    assert [m.kind for m, _ in c.layers] == ["attention", "delta", "parallel", "attention", "delta", "attention"]
    assert [ff for _, ff in c.layers] == [90, 70, 33, None, None, 40]
    a, d, p = (c.layers[i][0] for i in (0, 1, 2))
    assert (a.window, a.keep, a.softcap, a.dim_p, a.vdim_p) == (17, 3, 12.0, 32, 32)
    assert (d.taps, d.dim_p, d.vdim_p) == (3, 32, 48) and (p.right.inner, p.right.state_p, p.left.window) == (120, 32, 9)
    s = c.tensor_shapes()
    assert s["side.embed"] == (131, 72) and "l3.mix.k" not in s and "l3.mix.k.norm" not in s and s["l3.mix.q.b"] == (120,)
    assert s["l2.mix.right.in"] == (120 + 120 + 2 * 40 + 6, 72) and s["l2.mix.left.g"] == (3, 72) and "l2.mix.left.q.b" not in s
    assert "l3.norm2" not in s and s["l1.mix.q.conv"] == (48, 3) and s["l1.mix.v.conv"] == (160, 3)
    o = KemuzenConfig(M.MODELS["open"]).tensor_shapes()
    assert "side.embed" not in o and "l0.side.gate" not in o


def test_a_shared_cache_reaches_as_far_as_its_widest_user():
    from nvmai_amd.kemuzen import KemuzenConfig
    c = KemuzenConfig(M.MODELS["mixed"])
    assert [c.cache_of(i) for i in (0, 2, 3, 5)] == [0, 2, 0, 0] and c.reach(0) == (50, 70) and c.reach(2) == (9, 0)
    assert KemuzenConfig(M.MODELS["open"]).reach(0) == (0, 2)


@pytest.mark.parametrize("change,kind", [
    (lambda c: c["embedding"].pop("scale"), "indexCorrupt"), (lambda c: c["norm"].pop("eps"), "indexCorrupt"),
    (lambda c: c["layers"][0].update(type="other"), "unsupportedArch"),
    (lambda c: c["layers"][0]["mlp"].update(kind="routed"), "unsupportedArch"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "indexCorrupt"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "indexCorrupt"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=1), "indexCorrupt"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=4), "indexCorrupt"),
    (lambda c: c["layers"][5]["mixer"].update(kv_from=3), "indexCorrupt"),
    (lambda c: c["layers"][3]["mixer"].update(dim=24), "indexCorrupt"),
    (lambda c: c["layers"][2]["mixer"]["right"].update(norm_groups=7), "indexCorrupt"),
    (lambda c: c["layers"][2]["mixer"].pop("left_scale"), "indexCorrupt"),
    (lambda c: c["layers"][1]["mixer"].pop("conv"), "indexCorrupt")])
def test_config_refuses_what_it_does_not_know(change, kind):
    from nvmai_amd.gturbo import ModelError
    from nvmai_amd.kemuzen import KemuzenConfig
    c = copy(M.MODELS["mixed"])
    change(c)
    with pytest.raises(ModelError) as e:
        KemuzenConfig(c)
    assert e.value.kind == kind


def test_registry_knows_the_design(tmp_path):
    from nvmai_amd import registry
    write_model(tmp_path / "m", M.MODELS["ones"], M.weights(M.MODELS["ones"], 1))
    f = registry.family_of(str(tmp_path / "m"))
    assert f.name == "Kemuzen" and f.activations == ("bfloat16", "float32")


# ---- weight layout -------------------------------------------------------------------------------------------
class _Host:
    """A stand-in context: the layout runs on host tensors."""
    device, act = torch.device("cpu"), 0


@pytest.mark.parametrize("name", ["mixed", "ones", "wide"])
def test_padded_and_grouped_weights_hold_every_element(name):
    from nvmai_amd.kemuzen import KemuzenConfig, KemuzenWeights
    cfg = KemuzenConfig(M.MODELS[name])
    t = M.weights(M.MODELS[name], 3)
    w = KemuzenWeights(_Host, cfg, t.__getitem__, lambda n: t[n].shape)
    rng = np.random.default_rng(0)
    f = lambda v: v.double().numpy()
    x = rng.standard_normal(cfg.width)
    h = np.concatenate([x, np.zeros(cfg.width_p - cfg.width)])

    def same(got, heads, size, padded, want):
        got = got[:heads * padded].reshape(heads, padded)
        assert np.allclose(got[:, :size].ravel(), want) and not got[:, size:].any()
    for i, (m, ff) in enumerate(cfg.layers):
        L, p = w.layers[i], "l%d.mix." % i
        y, at = f(L["in_proj"]) @ h + (0.0 if L["in_bias"] is None else f(L["in_bias"])), L["at"]
        assert L["in_proj"].shape[1] % 64 == 0 and L["in_proj"].shape[0] % 16 == 0
        lin = lambda n, bias=False: f(t[p + n]) @ x + (f(t[p + n + ".b"]) if bias else 0.0)
        if m.kind == "delta":
            same(y[at["conv"]:], m.kv_heads, m.dim, m.dim_p, lin("q"))
            same(y[m.kv_heads * m.dim_p:], m.kv_heads, m.dim, m.dim_p, lin("k"))
            same(y[2 * m.kv_heads * m.dim_p:], m.heads, m.vdim, m.vdim_p, lin("v"))
            same(y[at["g"]:], m.heads, m.vdim, m.vdim_p, lin("g"))
            assert np.allclose(y[at["a"]:][:m.heads], lin("a")) and np.allclose(y[at["b"]:][:m.heads], lin("b"))
            conv = f(L["conv"])
            for tap in range(m.taps):
                same(conv[m.kv_heads * m.dim_p:, tap], m.kv_heads, m.dim, m.dim_p, f(t[p + "k.conv"])[:, tap])
                same(conv[2 * m.kv_heads * m.dim_p:, tap], m.heads, m.vdim, m.vdim_p, f(t[p + "v.conv"])[:, tap])
            outs = [("o", m.heads, m.vdim, m.vdim_p)]
        else:
            a, q = (m, "") if m.kind == "attention" else (m.left, "left.")
            same(y[at["q"]:], a.heads, a.dim, a.dim_p, lin(q + "q", m.kind == "attention"))
            if a.kv_from is None:
                same(y[at["k"]:], a.kv_heads, a.dim, a.dim_p, lin(q + "k", m.kind == "attention"))
                same(y[at["v"]:], a.kv_heads, a.vdim, a.vdim_p, lin(q + "v", m.kind == "attention"))
            else:
                assert L["k_norm"] is None
            outs = [(q + "o", a.heads, a.vdim, a.vdim_p)]
        if m.kind == "parallel":
            r = m.right
            z, xs, b, c, dt = np.split(lin("right.in"), np.cumsum([r.inner, r.inner, r.groups * r.state, r.groups * r.state]))
            assert np.allclose(y[at["gate"]:][:m.left.heads], lin("left.g")) and np.allclose(y[at["dt"]:][:r.heads], dt)
            same(y[at["conv"]:], r.groups, r.state, r.state_p, c)
            same(y[at["conv"] + r.groups * r.state_p:], r.groups, r.state, r.state_p, b)
            same(y[at["conv"] + 2 * r.groups * r.state_p:], r.heads, r.vdim, r.vdim_p, xs)
            same(y[at["z"]:], r.heads, r.vdim, r.vdim_p, z)
            bias = f(t[p + "right.conv.b"])
            same(f(L["conv_bias"]), r.groups, r.state, r.state_p, bias[r.inner + r.groups * r.state:])
            same(f(L["norm"]), r.heads, r.vdim, r.vdim_p, f(t[p + "right.norm"]))
            outs.append(("right.o", r.heads, r.vdim, r.vdim_p))
        o, col = f(L["o"]), 0
        for n, heads, size, padded in outs:
            part = o[:, col:col + heads * padded].reshape(cfg.width, heads, padded)
            assert np.array_equal(part[:, :, :size].reshape(cfg.width, -1), f(t[p + n])) and not part[:, :, size:].any()
            col += heads * padded
        assert not o[:, col:].any() and o.shape[1] % 64 == 0
        if ff is not None:
            y = f(L["gate_up"]) @ h
            assert np.allclose(y[0:2 * ff:2], f(t["l%d.mlp.gate" % i]) @ x) and np.allclose(y[1:2 * ff:2], f(t["l%d.mlp.up" % i]) @ x)
        if cfg.side:
            assert torch.equal(L["side_embed"], t["side.embed"][:, i * cfg.side:(i + 1) * cfg.side])


def test_weights_refuse_a_wrong_shape():
    from nvmai_amd.gturbo import ModelError
    from nvmai_amd.kemuzen import KemuzenConfig, KemuzenWeights
    cfg = KemuzenConfig(M.MODELS["open"])
    t = M.weights(M.MODELS["open"], 3)
    bad = dict(t, **{"l0.mix.k": t["l0.mix.k"][:-1]})
    with pytest.raises(ModelError):
        KemuzenWeights(_Host, cfg, bad.__getitem__, lambda n: bad[n].shape)


# ---- the oracle itself --------------------------------------------------------------------------------------
def test_oracle_continues_a_sequence_from_its_states():
    cfg = M.MODELS["mixed"]
    o = K.Oracle(cfg, numpy64(M.weights(cfg, 2)))
    toks = tokens(cfg, 40, 1)
    whole = o.forward(toks)
    states, out = o.new_states(), []
    for a, b in [(0, 2), (2, 25), (25, 26), (26, 40)]:
        out.append(o.forward(toks[a:b], a, states))
    assert np.allclose(np.concatenate(out), whole, atol=1e-12)


def _planted(change):
    cfg = M.MODELS["mixed"]
    t = numpy64(M.weights(cfg, 2))
    toks = tokens(cfg, 140, 1)
    off, tt = copy(cfg), dict(t)
    change(off, tt)
    return logit_error(K.Oracle(off, tt).forward(toks), K.Oracle(cfg, t).forward(toks)).max()


@pytest.mark.parametrize("layer", [0, 2, 3, 5])
@pytest.mark.parametrize("by", [1, -1])
def test_a_window_that_is_one_token_off_shows(layer, by):
    def change(c, t):
        m = c["layers"][layer]["mixer"]
        m.get("left", m)["mask"]["size"] += by
    assert _planted(change) > 5e-3


@pytest.mark.parametrize("layer,by", [(0, 1), (0, -1), (3, -1), (5, 1), (5, -1)])
def test_a_kept_token_too_many_or_too_few_shows(layer, by):
    assert _planted(lambda c, t: c["layers"][layer]["mixer"]["mask"].update(keep_first=M.MODELS["mixed"]["layers"][layer]["mixer"]["mask"]["keep_first"] + by)) > 5e-3


def test_other_planted_mistakes_show():
    def roll(name):
        return lambda c, t: t.update({name: np.roll(t[name], 1, axis=0)})
    for change in (lambda c, t: c["layers"][3]["mixer"].update(softcap=5.2), lambda c, t: c["embedding"].update(scale=2.05),
                   lambda c, t: c["layers"][2]["mixer"].update(left_scale=0.75), lambda c, t: c.update(logit_softcap=12.0),
                   roll("l2.mix.right.D"), roll("l2.mix.right.conv.b"), roll("l1.mix.dt_bias"), roll("l4.mix.A_log"), roll("l0.mix.v.b"),
                   roll("side.embed"), lambda c, t: t.update({"l1.mix.k.conv": t["l1.mix.k.conv"][:, ::-1]})):
        assert _planted(change) > 2e-3


def test_oracle_pieces():
    assert K.visible(6, {"size": 3, "keep_first": 2}) == [0, 1, 4, 5, 6] and K.visible(2, None) == [0, 1, 2] and K.visible(1, {"size": 1}) == [1]
    s = K.sinusoid(3, 5)
    assert np.allclose(s, [np.sin(3), np.cos(3), np.sin(3 * 1e4 ** -0.4), np.cos(3 * 1e4 ** -0.4), np.sin(3 * 1e4 ** -0.8)])
    assert np.allclose([K.slope(h, 8) for h in (0, 7)], [0.5, 2.0 ** -8]) and K.slope(2, 3) == 2.0 ** -8
    assert np.allclose(K.gelu_tanh(np.array([0.0, 1.0, -1.0])), [0.0, 0.841192, -0.158808], atol=1e-6)
    past, w = [], np.array([[1.0, 2.0, 3.0]])
    outs = [K.short_conv(past, np.array([v]), w, np.array([0.5])) for v in (1.0, 10.0, 100.0)]
    assert np.allclose(np.concatenate(outs), K.silu(np.array([3.5, 32.5, 321.5])))
    assert np.allclose(K.softplus(np.array([-800.0, 0.0, 800.0])), [0.0, np.log(2.0), 800.0])
    # one key written and read back: the delta rule returns what it stored
    S = np.zeros((2, 3))
    k, v = np.array([0.6, 0.8]), np.array([1.0, -2.0, 3.0])
    S, o = K.delta_step(S, k, k, v, 1.0, 0.9)
    assert np.allclose(o, v)
    S, o = K.delta_step(S, k, k, -v, 1.0, 1.0)
    assert np.allclose(o, -v)
    S, y = K.ssd_step(np.ones((2, 1)), np.array([2.0]), np.array([1.0, 0.0]), np.array([1.0, 1.0]), 0.5, 2.0, 10.0)
    assert np.allclose(y, 2.0 * np.exp(-1.0) + 1.0 + 20.0)
