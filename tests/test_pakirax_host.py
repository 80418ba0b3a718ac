"""Host side of the Pakirax model and of the layers around it (no GPU): configuration, registry, the safetensors
container, weight layout, sessions, command line, and the oracle's own identities."""
import json
import os
import struct

import numpy as np
import pytest
import torch

import pakirax_models as M
import pakirax_oracle as P


# ---- configuration and registry ---------------------------------------------------------------------
def test_config_reads_every_layer_by_itself():
    from nvmai_amd.pakirax import PakiraxConfig
    c = PakiraxConfig(M.MODELS["mixed"])
    assert [m.kind for m, _ in c.layers] == ["latent_attention", "gla", "latent_attention", "gla", "latent_attention"]
    assert [ff for _, ff in c.layers] == [90, 70, None, None, 33]
    a, b = c.layers[0][0], c.layers[4][0]
    assert (a.window, a.dim_p, a.rot_p, a.vdim_p, a.rank_p, b.window, b.rot_base) == (17, 32, 16, 32, 64, 5, 500.0)
    s = c.tensor_shapes(lambda i: 6 + i)
    assert s["l1.mix.a1"] == (7, 72) and s["l0.mix.uq"] == (96, 36) and "l2.norm2" not in s and s["l4.mlp.down"] == (72, 33)


@pytest.mark.parametrize("change,kind", [
    (lambda c: c.pop("residual_mult"), "indexCorrupt"), (lambda c: c["norm"].pop("eps"), "indexCorrupt"),
    (lambda c: c["layers"][0].update(type="other"), "unsupportedArch"),
    (lambda c: c["layers"][0]["mlp"].update(kind="routed"), "unsupportedArch"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=40), "indexCorrupt"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "indexCorrupt"),
    (lambda c: c["layers"][1]["mixer"].pop("tau"), "indexCorrupt")])
def test_config_refuses_what_it_does_not_know(change, kind):
    from nvmai_amd.gturbo import ModelError
    from nvmai_amd.pakirax import PakiraxConfig
    c = json.loads(json.dumps(M.MODELS["mixed"]))
    change(c)
    with pytest.raises(ModelError) as e:
        PakiraxConfig(c)
    assert e.value.kind == kind


def test_registry_chooses_by_the_directory(tmp_path):
    from nvmai_amd import registry
    with pytest.raises(registry.UnknownModel):
        registry.family_of(str(tmp_path))
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Other"}))
    with pytest.raises(registry.UnknownModel):
        registry.family_of(str(tmp_path))
    (tmp_path / "config.json").write_text(json.dumps(M.MODELS["mixed"]))
    assert registry.family_of(str(tmp_path)).name == "Pakirax"
    with pytest.raises(registry.UnknownModel):
        registry.open_model(str(tmp_path), "float16")
    (tmp_path / "manifest.json").write_text("{}")
    assert registry.family_of(str(tmp_path)).name == "hybrid-moe"


# ---- safetensors ------------------------------------------------------------------------------------------
def test_safetensors_round_trip_and_corrupt_files(tmp_path):
    from nvmai_amd.safetensors_file import SafetensorsError, SafetensorsFile, write_safetensors
    t = {"a": torch.randn(3, 5).to(torch.bfloat16), "b.c": torch.arange(7, dtype=torch.int32), "s": torch.tensor(2.5), "e": torch.zeros((0, 4))}
    path = str(tmp_path / "m.safetensors")
    write_safetensors(path, t)
    f = SafetensorsFile(path)
    assert set(f.entries) == set(t) and f.shape("a") == (3, 5) and "x" not in f
    assert all(torch.equal(f.tensor(n), t[n]) and f.tensor(n).dtype == t[n].dtype for n in t)
    raw = open(path, "rb").read()
    n = struct.unpack("<Q", raw[:8])[0]
    bad = tmp_path / "bad.safetensors"
    for data in (raw[:5], struct.pack("<Q", 1 << 40) + raw[8:], raw[:-3], raw[:8 + n].replace(b'"shape": [3, 5]', b'"shape": [3, 6]') + raw[8 + n:]):
        bad.write_bytes(data)
        with pytest.raises(SafetensorsError):
            SafetensorsFile(str(bad))


def test_safetensors_agrees_with_the_installed_reader(tmp_path):
    st = pytest.importorskip("safetensors.torch")
    from nvmai_amd.safetensors_file import SafetensorsFile, write_safetensors
    t = {"w": torch.randn(4, 6).to(torch.bfloat16), "i": torch.arange(5, dtype=torch.int32)}
    write_safetensors(str(tmp_path / "a"), t)
    st.save_file(t, str(tmp_path / "b"))
    assert all(torch.equal(st.load_file(str(tmp_path / "a"))[n], t[n]) for n in t)
    assert all(torch.equal(SafetensorsFile(str(tmp_path / "b")).tensor(n), t[n]) for n in t)


# ---- weight layout -------------------------------------------------------------------------------------------
class _Host:
    """A stand-in context: the layout runs on host tensors."""
    device, act = torch.device("cpu"), 0


def test_padded_and_grouped_weights_hold_every_element():
    from nvmai_amd.pakirax import PakiraxConfig, PakiraxWeights
    cfg = PakiraxConfig(M.MODELS["mixed"])
    t = M.weights(M.MODELS["mixed"], 3)
    w = PakiraxWeights(_Host, cfg, t.__getitem__, lambda n: t[n].shape)
    rng = np.random.default_rng(0)
    f = lambda v: v.double().numpy()
    for i, (m, ff) in enumerate(cfg.layers):
        L, p = w.layers[i], "l%d.mix." % i
        h = np.zeros(cfg.width_p)
        h[:cfg.width] = rng.standard_normal(cfg.width)
        y = f(L["in_proj"]) @ h
        assert L["in_proj"].shape[1] % 64 == 0 and L["in_proj"].shape[0] % 16 == 0
        if m.kind == "gla":
            for n, d, dp in (("q", m.dim, m.dim_p), ("k", m.dim, m.dim_p), ("v", m.vdim, m.vdim_p), ("g", m.vdim, m.vdim_p)):
                got = y[L["at"][n]:][:m.heads * dp].reshape(m.heads, dp)
                assert np.allclose(got[:, :d].ravel(), f(t[p + n]) @ h[:cfg.width]) and not got[:, d:].any()
            a1 = y[L["at"]["a1"]:]
            assert np.allclose(f(L["a2"]).reshape(m.heads, m.dim_p, -1)[:, :m.dim].reshape(m.heads * m.dim, -1) @ a1[:L["rank"]],
                               f(t[p + "a2"]) @ (f(t[p + "a1"]) @ h[:cfg.width]))
        else:
            assert np.allclose(y[L["at"]["g"]:][:m.heads], f(t[p + "g"]) @ h[:cfg.width])
            kv = f(t[p + "dkv"]) @ h[:cfg.width]
            assert np.allclose(y[L["at"]["kv"]:][:m.kv_rank], kv[:m.kv_rank]) and np.allclose(y[L["at"]["rope"]:][:m.rot_dim], kv[m.kv_rank:])
            uq = f(L["uq"]).reshape(m.heads, m.dim_p + m.rot_p, -1)
            want = f(t[p + "uq"]).reshape(m.heads, m.dim + m.rot_dim, -1)
            assert np.array_equal(uq[:, :m.dim, :m.q_rank], want[:, :m.dim]) and np.array_equal(uq[:, m.dim_p:m.dim_p + m.rot_dim, :m.q_rank], want[:, m.dim:])
            assert abs(uq).sum() == pytest.approx(abs(want).sum())
        o = f(L["o"])[:, :m.heads * m.vdim_p].reshape(cfg.width, m.heads, m.vdim_p)
        assert np.array_equal(o[:, :, :m.vdim].reshape(cfg.width, -1), f(t[p + "o"])) and not o[:, :, m.vdim:].any()


def test_weights_refuse_a_wrong_shape_or_type():
    from nvmai_amd.gturbo import ModelError
    from nvmai_amd.pakirax import PakiraxConfig, PakiraxWeights
    cfg = PakiraxConfig(M.MODELS["gla_only"])
    t = M.weights(M.MODELS["gla_only"], 3)
    bad = dict(t, **{"l0.mix.k": t["l0.mix.k"][:-1]})
    with pytest.raises(ModelError):
        PakiraxWeights(_Host, cfg, bad.__getitem__, lambda n: bad[n].shape)
    bad = dict(t, **{"embed": t["embed"].float()})
    with pytest.raises(ModelError):
        PakiraxWeights(_Host, cfg, bad.__getitem__, lambda n: bad[n].shape)


# ---- sessions and generation over a stand-in driver --------------------------------------------------------
class _Driver:
    """Counts instead of computing: a row is (sum of what the slot was fed, tokens fed)."""
    batch, max_context = 2, 64

    class ctx:
        device = torch.device("cpu")

    def __init__(self):
        self.sums, self.calls = [None, None], []

    def reset(self, slot):
        self.sums[slot] = 0

    def prefill_rows(self, ids, slot, at, want):
        rows = []
        for t in ids.tolist():
            self.sums[slot] += t
            rows.append(self.sums[slot])
        self.calls.append(("prefill", slot, at, len(rows)))
        want = [len(rows) - 1] if want is None else want
        return torch.tensor([[float(rows[p])] for p in want]) if len(want) else None

    def decode_rows(self, slots, positions, tokens):
        for s, t in zip(slots, tokens):
            self.sums[s] += t
        self.calls.append(("decode", tuple(slots), tuple(positions)))
        return torch.tensor([[float(self.sums[s])] for s in slots])


def test_session_gives_slots_back_and_starts_them_anew():
    from nvmai_amd.generate import Session
    d = _Driver()
    s = Session(d)
    assert s.feed("a", [1, 2, 3], [0, 2]).ravel().tolist() == [1.0, 6.0] and s.length("a") == 3
    assert s.feed("a", [4], [0]).item() == 10.0 and s.feed("a", [5], []) is None and s.length("a") == 5
    assert s.feed("b", [7]).item() == 7.0                      # a first token alone is a prompt
    with pytest.raises(RuntimeError):
        s.feed("c", [1])
    assert s.decode(["b", "a"], [1, 2]).ravel().tolist() == [8.0, 17.0]
    s.end("a")
    assert "a" not in s and s.feed("c", [9, 9]).item() == 18.0   # slot 0 again, from zero
    assert d.calls[-1] == ("prefill", 0, 0, 2) and ("decode", (1, 0), (1, 5)) in d.calls


def test_portions_longer_than_a_chunk_are_cut_and_wanted_rows_found():
    from nvmai_amd.decoder import StepDecoder

    class D(StepDecoder):
        max_chunk = 4

        def __init__(self):
            self.max_context, self.cuts, self.buf = 100, [], torch.zeros(4, 1)

        def _prefill_chunk_rows(self, tokens, b, start):
            self.cuts.append((start, tokens.numel()))
            rows = self.buf[:tokens.numel()]
            rows.copy_(tokens[:, None].float())              # one buffer for every chunk
            return rows
    d = D()
    ids = torch.arange(10, 21, dtype=torch.int32)
    assert d.prefill_rows(ids, 0, 5, [10, 0, 3, 4]).ravel().tolist() == [20.0, 10.0, 13.0, 14.0]
    assert d.cuts == [(5, 4), (9, 4), (13, 3)]
    assert d.prefill_chunked(ids).item() == 20.0 and d.prefill_rows(ids, want=[]) is None
    for bad in (lambda: d.prefill_rows(ids, want=[11]), lambda: d.prefill_rows(ids[:0]), lambda: d.prefill_rows(ids, 0, 95)):
        with pytest.raises(ValueError):
            bad()


def test_command_line_parses():
    from nvmai_amd import cli
    a = cli.parser().parse_args(["replay", "--model", "m", "--dtype", "float32", "--out", "o", "--max-tokens", "9"])
    assert (a.command, a.model, a.dtype, a.out, a.max_tokens, a.slots) == ("replay", "m", "float32", "o", 9, 1)
    a = cli.parser().parse_args(["generate", "--model", "m", "--prompt", "1,2", "--prompt", "3"])
    assert [cli._ids(p) for p in a.prompt] == [[1, 2], [3]] and a.temperature == 0.0


def test_part_library_names_existing_sources():
    from nvmai_amd import build
    for part, names in build.PARTS.items():
        assert build.part_path(part) != build.LIB
        for n in names:
            assert os.path.exists(os.path.join(build.CSRC, n + ".hip"))


# ---- the oracle itself --------------------------------------------------------------------------------------
def test_oracle_continues_a_sequence_from_its_states():
    cfg = M.MODELS["mixed"]
    o = P.Oracle(cfg, M.numpy64(M.weights(cfg, 2)))
    toks = M.tokens(cfg, 40, 1)
    whole = o.forward(toks)
    states, out = o.new_states(), []
    for a, b in [(0, 2), (2, 25), (25, 26), (26, 40)]:
        out.append(o.forward(toks[a:b], a, states))
    assert np.allclose(np.concatenate(out), whole, atol=1e-12)


def test_oracle_sees_a_window_that_is_one_token_off():
    cfg = M.MODELS["mixed"]
    t = M.numpy64(M.weights(cfg, 2))
    toks = M.tokens(cfg, 60, 1)
    want = P.Oracle(cfg, t).forward(toks)
    for layer in (0, 2, 4):
        off = json.loads(json.dumps(cfg))
        off["layers"][layer]["mixer"]["mask"]["size"] += 1
        assert M.logit_error(P.Oracle(off, t).forward(toks), want).max() > 1e-2
    off = json.loads(json.dumps(cfg))
    off["layers"][1]["mixer"]["tau"] *= 1.02
    assert M.logit_error(P.Oracle(off, t).forward(toks), want).max() > 1e-4


def test_oracle_pieces():
    x = np.array([1.0, 2.0, 3.0, 4.0, 5.0, 6.0])
    r = P.rotate_half(x, 2, 100.0, 4)
    a0, a1 = 2.0, 2.0 / 10.0
    assert np.allclose(r, [np.cos(a0) - 3 * np.sin(a0), 2 * np.cos(a1) - 4 * np.sin(a1), 3 * np.cos(a0) + np.sin(a0),
                           4 * np.cos(a1) + 2 * np.sin(a1), 5, 6])
    assert list(P.window_keys(10, 3)) == [8, 9, 10] and list(P.window_keys(1, 3)) == [0, 1] and list(P.window_keys(4, None)) == [0, 1, 2, 3, 4]
    assert np.allclose(P.decay(np.array([-800.0, 0.0, 800.0]), 16.0), [np.exp(-50.0), 0.5 ** (1 / 16), 1.0])
    assert np.allclose(P.gelu_erf(np.array([0.0, 1.0, -1.0])), [0.0, 0.8413447460685429, -0.15865525393145707])
