"""Kemuzen: a decoder-only language model whose layers mix tokens by windowed attention with kept first tokens, by the
gated delta rule, or by windowed attention and a state-space recurrence side by side; norms stand on the sublayers'
outputs only, and every layer ends with an input of its own per token.  Configuration, weights and step driver; what the
driver shares with the other dense models is in dense_model.py.

With N the sublayers' norms, a layer adds N(M x), then N(F x) where it has a feed-forward F, then N(W_p (gelu(W_g x) . e)) to the
residual x, each from x as the one before left it; e is the layer's part of the token's side vector.  The residual is
32-bit and starts as the scaled embedding plus a sinusoid of the position.  Every size and constant comes from config.json or from a tensor's shape, layer by layer.

Weights are laid out for one launch per projection group (a mixer's projections of its input are rows of one matrix, both
mixers' of a parallel layer; its two output projections are columns of one) and padded with zeros so that the kernels see
multiples of 16 (heads; 32 for attention's keys) and 64 (the k of a product); real counts go with them where a norm needs
them."""
import torch

from . import ops
from .dense_model import DenseDecoder, bf16_reader, blocks_of, check_shapes, need, open_directory, pad_columns, up
from .gturbo import ModelError


def _divides(where, heads, groups):
    if heads < 1 or groups < 1 or heads % groups:
        raise ModelError("indexCorrupt", "config.json: %s: %d heads over %d" % (where, heads, groups))


class Attention:
    """Grouped-query attention over a window and the first tokens; kv_from: the layer whose keys and values it uses."""

    def __init__(self, m, where):
        self.heads, self.kv_heads, self.dim, self.vdim, self.scale = need(m, where, "heads", "kv_heads", "dim", "vdim", "scale")
        mask = m.get("mask")
        self.window, self.keep = (int(mask["size"]), int(mask.get("keep_first", 0))) if mask else (0, 0)
        self.softcap, self.kv_from = float(m.get("softcap") or 0.0), m.get("kv_from")
        self.dim_p, self.vdim_p = up(self.dim, 32), up(self.vdim, 16)
        _divides(where, self.heads, self.kv_heads)
        if (mask and self.window < 1) or self.keep < 0:
            raise ModelError("indexCorrupt", "config.json: %s: mask out of range" % where)

    def shapes(self, width, bias, gate):
        q, k, v = self.heads * self.dim, self.kv_heads * self.dim, self.kv_heads * self.vdim
        out = {"q": (q, width), "q.norm": (self.dim,), "o": (width, self.heads * self.vdim)}
        if self.kv_from is None:
            out.update({"k": (k, width), "k.norm": (self.dim,), "v": (v, width)})
        if bias:
            out.update({n + ".b": out[n][:1] for n in ("q", "k", "v", "o") if n in out})
        if gate:
            out["g"] = (self.heads, width)
        return out

    def projections(self, t):
        """(rows of the input projection, where each part starts in them): t(name) -> its matrix or vector."""
        rows = [blocks_of(t("q"), 0, [(self.heads, self.dim, self.dim_p)])]
        at = dict(q=0, k=self.heads * self.dim_p, v=(self.heads + self.kv_heads) * self.dim_p)
        if self.kv_from is None:
            rows += [blocks_of(t("k"), 0, [(self.kv_heads, self.dim, self.dim_p)]), blocks_of(t("v"), 0, [(self.kv_heads, self.vdim, self.vdim_p)])]
        return rows, at


class AttentionLayer(Attention):
    kind = "attention"

    def tensors(self, width):
        return self.shapes(width, True, False)


class DeltaLayer:
    kind = "delta"

    def __init__(self, m, where):
        self.heads, self.kv_heads, self.dim, self.vdim, self.taps = need(m, where, "heads", "kv_heads", "dim", "vdim", "conv")
        self.dim_p, self.vdim_p = up(self.dim, 16), up(self.vdim, 16)
        _divides(where, self.heads, self.kv_heads)

    def tensors(self, width):
        kd, vd, H = self.kv_heads * self.dim, self.heads * self.vdim, self.heads
        return {"q": (kd, width), "q.conv": (kd, self.taps), "k": (kd, width), "k.conv": (kd, self.taps), "v": (vd, width),
                "v.conv": (vd, self.taps), "b": (H, width), "A_log": (H,), "norm": (self.vdim,), "a": (H, width), "dt_bias": (H,),
                "g": (vd, width), "o": (width, vd)}


class Ssd:
    """The state-space mixer: inner = heads * vdim channels, `groups` shared inputs and outputs of the state."""

    def __init__(self, m, where):
        self.heads, self.vdim, self.state, self.groups, self.taps, self.norm_groups = \
            need(m, where, "heads", "vdim", "state", "groups", "conv", "norm_groups")
        self.state_p, self.vdim_p, self.inner = up(self.state, 16), up(self.vdim, 16), self.heads * self.vdim
        _divides(where, self.heads, self.groups)
        _divides(where + " norm", self.inner, self.norm_groups)

    def shapes(self, width):
        gn, H = self.groups * self.state, self.heads
        channels = self.inner + 2 * gn
        return {"in": (self.inner + channels + H, width), "conv": (channels, self.taps), "conv.b": (channels,), "dt_bias": (H,),
                "A_log": (H,), "D": (H,), "norm": (self.inner,), "o": (width, self.inner)}

    def channels(self, v):
        """Rows [x | B | C] of a tensor as the kernels take them: [C | B | x], padded."""
        gn = self.groups * self.state
        x, b, c = v.split([self.inner, gn, gn])
        pad = lambda t: blocks_of(t, 0, [(self.groups, self.state, self.state_p)])
        return torch.cat([pad(c), pad(b), blocks_of(x, 0, [(self.heads, self.vdim, self.vdim_p)])])


class ParallelLayer:
    kind = "parallel"

    def __init__(self, m, where):
        left, right, self.left_scale, self.right_scale = need(m, where, "left", "right", "left_scale", "right_scale")
        self.left, self.right = Attention(left, where + " left"), Ssd(right, where + " right")
        if self.left.kv_from is not None:
            raise ModelError("unsupportedArch", "%s: keys of another layer in a parallel mixer" % where)

    def tensors(self, width):
        out = {"left." + n: s for n, s in self.left.shapes(width, False, True).items()}
        out.update({"right." + n: s for n, s in self.right.shapes(width).items()})
        return out


MIXERS = {c.kind: c for c in (AttentionLayer, DeltaLayer, ParallelLayer)}


class KemuzenConfig:
    """config.json, checked.  layers: one (mixer, ff or None) per layer."""

    def __init__(self, config):
        self.vocab, self.width, embedding, norm, layers = need(config, "the model", "vocab", "width", "embedding", "norm", "layers")
        self.eps, = need(norm, "norm", "eps")
        self.embed_scale, = need(embedding, "embedding", "scale")
        self.hidden = self.width
        self.width_p = up(self.width, 64)
        self.logit_softcap = float(config.get("logit_softcap") or 0.0)
        self.side = int(config["token_side"]["dim"]) if config.get("token_side") else 0
        self.layers = []
        for i, e in enumerate(layers):
            where = "layer %d" % i
            kind, mixer = need(e, where, "type", "mixer")
            if kind not in MIXERS:
                raise ModelError("unsupportedArch", "%s: mixer %s" % (where, kind))
            ff = None
            if e.get("mlp") is not None:
                mlp_kind, ff = need(e["mlp"], where + "'s mlp", "kind", "ff")
                if mlp_kind != "dense":
                    raise ModelError("unsupportedArch", "%s: feed-forward %s" % (where, mlp_kind))
            m = MIXERS[kind](mixer, where)
            if kind == "attention" and m.kv_from is not None:
                j = m.kv_from
                owner = self.layers[j][0] if 0 <= j < i else None
                if owner is None or owner.kind != "attention" or owner.kv_from is not None or \
                        (owner.kv_heads, owner.dim, owner.vdim) != (m.kv_heads, m.dim, m.vdim):
                    raise ModelError("indexCorrupt", "config.json: %s cannot use layer %s's keys" % (where, j))
            self.layers.append((m, ff))

    def cache_of(self, i):
        """The layer whose cache layer i looks at."""
        m = self.layers[i][0]
        return i if m.kind != "attention" or m.kv_from is None else m.kv_from

    def reach(self, i):
        """(window, kept first positions) that layer i's cache has to hold for every layer that looks at it; window 0: all."""
        users = [m.left if m.kind == "parallel" else m for j, (m, _) in enumerate(self.layers)
                 if m.kind != "delta" and self.cache_of(j) == i]
        return 0 if any(m.window == 0 for m in users) else max(m.window for m in users), max(m.keep for m in users)

    def tensor_shapes(self):
        """Name -> shape of every tensor."""
        W = self.width
        out = {"embed": (self.vocab, W), "final.norm": (W,)}
        if self.side:
            out["side.embed"] = (self.vocab, len(self.layers) * self.side)
        for i, (m, ff) in enumerate(self.layers):
            p = "l%d." % i
            out[p + "norm1"] = (W,)
            out.update({p + "mix." + n: s for n, s in m.tensors(W).items()})
            if ff is not None:
                out.update({p + "norm2": (W,), p + "mlp.gate": (ff, W), p + "mlp.up": (ff, W), p + "mlp.down": (W, ff)})
            if self.side:
                out.update({p + "side.gate": (self.side, W), p + "side.proj": (W, self.side), p + "side.norm": (W,)})
        return out

    def matrix_elements(self):
        """Elements of every matrix a token is multiplied by, the logits' included."""
        return sum(s[0] * s[1] for n, s in self.tensor_shapes().items() if len(s) == 2 and not n.endswith("conv") and n != "side.embed")

    def _mixers(self):
        for m, _ in self.layers:
            yield from ((m.left, m.right) if m.kind == "parallel" else (m,))

    def bytes_per_token(self, batch=1, context=32768, act_bytes=2):
        """Algorithmic HBM bytes of one decode step divided by the batch: every matrix once, recurrent states read and
        written, the keys and values the windows reach."""
        own = 0
        for m in self._mixers():
            if isinstance(m, Attention):
                own += act_bytes * (min(context, m.window + m.keep) if m.window else context) * m.kv_heads * (m.dim + m.vdim)
            else:
                own += 2 * 4 * m.heads * (m.state if isinstance(m, Ssd) else m.dim) * m.vdim
        return 2 * self.matrix_elements() / batch + own

    def prefill_flops(self, tokens):
        """Useful flops of a prompt of `tokens`: 2 per matrix element and token (the logits of one token), the pairs
        inside the windows, the recurrences' products (two for the state-space form, three for the delta rule)."""
        total = 2.0 * tokens * (self.matrix_elements() - self.vocab * self.width) + 2.0 * self.vocab * self.width
        for m in self._mixers():
            if isinstance(m, Attention):
                w = min(m.window or tokens, tokens)
                total += 2.0 * m.heads * (m.dim + m.vdim) * (w * (w + 1) / 2 + (tokens - w) * (w + min(m.keep, w)))
            elif isinstance(m, Ssd):
                total += 4.0 * tokens * m.heads * m.state * m.vdim
            else:
                total += 6.0 * tokens * m.heads * m.dim * m.vdim
        return total


class KemuzenWeights:
    """Device tensors of a model, padded and grouped.  source(name) -> BF16 tensor; shape(name) -> its shape."""

    def __init__(self, ctx, cfg, source, shape):
        self.ctx, self.cfg = ctx, cfg
        check_shapes(cfg.tensor_shapes(), shape)
        t, cols = bf16_reader(ctx, source), pad_columns
        self.embed = cols(t("embed")).contiguous()
        self.final_norm = t("final.norm").contiguous()
        side = t("side.embed").contiguous() if cfg.side else None
        self.layers = []
        for i, (m, ff) in enumerate(cfg.layers):
            p = "l%d." % i
            w = dict(norm1=t(p + "norm1").contiguous())
            w.update(getattr(self, "_" + m.kind)(m, lambda n: t(p + "mix." + n)))
            if ff is not None:
                # rows of the two matrices in turn: one launch makes silu(gate) * up
                gate, up_ = (blocks_of(t(p + "mlp." + n), 0, [(1, ff, up(ff, 64))]) for n in ("gate", "up"))
                w.update(norm2=t(p + "norm2").contiguous(), gate_up=cols(torch.stack([gate, up_], 1).flatten(0, 1)).contiguous(),
                         down=cols(t(p + "mlp.down")).contiguous())
            if cfg.side:
                w.update(side_gate=cols(t(p + "side.gate")).contiguous(), side_proj=cols(t(p + "side.proj")).contiguous(),
                         side_norm=t(p + "side.norm").contiguous(), side_embed=side[:, i * cfg.side:(i + 1) * cfg.side])
            self.layers.append(w)

    @staticmethod
    def _norms(m, t):
        pad = lambda n: blocks_of(t(n), 0, [(1, m.dim, m.dim_p)]).contiguous()
        return dict(q_norm=pad("q.norm"), k_norm=pad("k.norm") if m.kv_from is None else None)

    @staticmethod
    def _stack(rows, at, **more):
        """One matrix (or vector) of `rows` and the places of further parts behind them, rounded up to 16 rows."""
        n = sum(r.shape[0] for r in rows)
        for name, r in more.items():
            at[name] = n
            rows.append(r)
            n += r.shape[0]
        return blocks_of(torch.cat(rows), 0, [(1, n, up(n, 16))]), at

    def _attention(self, m, t):
        rows, at = m.projections(t)
        bias, _ = m.projections(lambda n: t(n + ".b"))
        w, at = self._stack(rows, at)
        b, _ = self._stack(bias, {})
        o = blocks_of(t("o"), 1, [(m.heads, m.vdim, m.vdim_p)], up(m.heads * m.vdim_p, 64))
        return dict(self._norms(m, t), in_proj=pad_columns(w).contiguous(), in_bias=b.contiguous(), at=at, o=o.contiguous(), o_bias=t("o.b").contiguous())

    def _delta(self, m, t):
        keys = lambda n: blocks_of(t(n), 0, [(m.kv_heads, m.dim, m.dim_p)])
        values = lambda n: blocks_of(t(n), 0, [(m.heads, m.vdim, m.vdim_p)])
        w, at = self._stack([keys("q"), keys("k"), values("v")], dict(conv=0), g=values("g"), b=t("b"), a=t("a"))
        return dict(in_proj=pad_columns(w).contiguous(), in_bias=None, at=at, conv=torch.cat([keys("q.conv"), keys("k.conv"), values("v.conv")]).contiguous(),
                    conv_bias=None, a_log=t("A_log").contiguous(), dt_bias=t("dt_bias").contiguous(), skip=None,
                    norm=blocks_of(t("norm"), 0, [(1, m.vdim, m.vdim_p)]).contiguous(),
                    o=blocks_of(t("o"), 1, [(m.heads, m.vdim, m.vdim_p)], up(m.heads * m.vdim_p, 64)).contiguous())

    def _parallel(self, m, t):
        a, r = m.left, m.right
        lt, rt = (lambda n: t("left." + n)), (lambda n: t("right." + n))
        heads = lambda v: blocks_of(v, 0, [(r.heads, r.vdim, r.vdim_p)])
        z, xbc, dt = rt("in").split([r.inner, r.inner + 2 * r.groups * r.state, r.heads])
        rows, at = a.projections(lt)
        w, at = self._stack(rows, at, gate=lt("g"), conv=r.channels(xbc), z=heads(z), dt=dt)
        left, right = (blocks_of(tt("o"), 1, [(x.heads, x.vdim, x.vdim_p)]) for tt, x in ((lt, a), (rt, r)))
        o = torch.cat([left, right], 1)
        return dict(self._norms(a, lt), in_proj=pad_columns(w).contiguous(), in_bias=None, at=at, conv=r.channels(rt("conv")).contiguous(),
                    conv_bias=r.channels(rt("conv.b")).contiguous(), a_log=rt("A_log").contiguous(), dt_bias=rt("dt_bias").contiguous(),
                    skip=rt("D").contiguous(), norm=heads(rt("norm")).contiguous(), o=pad_columns(o).contiguous())

    @classmethod
    def from_directory(cls, ctx, path):
        """(config, weights) of a folder with config.json and model.safetensors."""
        cfg, tensor, shape = open_directory(path, KemuzenConfig)
        return cfg, cls(ctx, cfg, tensor, shape)

    @classmethod
    def random(cls, ctx, cfg, seed=1234):
        """Random-init weights on the device, scaled so that activations stay of order one."""
        gen = torch.Generator(device=ctx.device).manual_seed(seed)
        shapes = cfg.tensor_shapes()

        def source(name):
            s = shapes[name]
            v = torch.empty(s, dtype=torch.float32, device=ctx.device)
            if len(s) == 1:
                v.normal_(0.0, 0.1, generator=gen)
                if name.endswith(("q.norm", "k.norm", "mix.norm", "right.norm", "side.norm", ".D")):
                    v += 1.0
                elif name.endswith("dt_bias"):
                    v -= 3.0
            else:
                v.normal_(0.0, s[1] ** -0.5, generator=gen)
            return v.to(torch.bfloat16)
        return cls(ctx, cfg, source, lambda n: shapes[n])


class KemuzenDecoder(DenseDecoder):
    """Prompt portions and decode steps of a Kemuzen model.  A ring holds the widest window of the layers that look at it
    beside one portion of max_chunk tokens, and the first tokens for good, so a layer's cache does not grow with the context."""
    long_f32 = ("residual", "delta", "proj", "scan")

    def __init__(self, ctx, cfg, weights, batch=1, max_context=32768, max_chunk=2048):
        super().__init__(ctx, cfg, weights, batch, max_context, max_chunk)
        self.attention, self.scans, self.states, self.caches = {}, {}, {}, {}
        self.inv_freq = ops.sinusoid_frequencies(cfg.width, ctx.device)
        for i, (m, _) in enumerate(cfg.layers):
            at = weights.layers[i]["at"]
            a, r = (m.left, m.right) if m.kind == "parallel" else (m, None) if m.kind == "attention" else (None, m)
            for c in self.contexts:
                if a is not None:
                    self.attention[i, c] = ops.WindowAttention(c, a.heads, a.dim, a.scale, a.window, cfg.eps, min(a.keep, max_context), a.softcap,
                                                               alibi=m.kind == "parallel")
                if m.kind == "delta":
                    self.scans[i, c] = ops.HeadScan(c, ops.SCAN_DELTA, m.heads, m.kv_heads, m.dim_p, m.vdim_p, m.taps, at["conv"], at["a"], at["b"],
                                                    m.dim ** -0.5)
                elif m.kind == "parallel":
                    self.scans[i, c] = ops.HeadScan(c, ops.SCAN_SSD, r.heads, r.groups, r.state_p, r.vdim_p, r.taps, at["conv"], at["dt"])
            if r is not None:
                self.states[i] = self.scans[i, ctx].new_state(batch)
            if a is not None:
                owner = cfg.cache_of(i)
                if owner not in self.caches:
                    window, keep = cfg.reach(owner)
                    capacity = min(max_context, window + self.max_chunk - 1) if window else max_context
                    self.caches[owner] = ops.KvRing(ctx, batch, a.kv_heads, a.dim_p, a.vdim_p, capacity, min(keep, max_context))
                self.caches[i] = self.caches[owner]

    # -- mixers: the layer's input in, the sublayer's output as 32-bit rows ---------------------------------
    def _window(self, ctx, i, a, proj, rows_at, out, gate=None, out_scale=1.0):
        """Attention of layer i from its projected rows into the first columns of out."""
        w, T = self.w.layers[i], proj.shape[0]
        op, cache, at = self.attention[i, ctx], self.caches[i], w["at"]
        q = self._buf("q", T, a.heads * a.dim_p, cache.k.dtype)
        op.encode_epilogue(proj, at["q"], at["k"], at["v"], w["q_norm"], w["k_norm"], q, cache, rows_at)
        op.encode(q, cache, rows_at, out, gate, out_scale)

    def _scan(self, ctx, i, proj, rows_at, heads, vdim_p):
        w = self.w.layers[i]
        T = proj.shape[0]
        y = self._buf("scan", T, heads * vdim_p, torch.float32).view(heads, T, vdim_p)         # head by head
        return self.scans[i, ctx].encode(proj, w["conv"], w["conv_bias"], w["a_log"], w["dt_bias"], w["skip"], *self.states[i], rows_at, y)

    def _mix(self, ctx, i, h, rows_at):
        m, w, T = self.cfg.layers[i][0], self.w.layers[i], h.shape[0]
        proj = ops.dense_linear(ctx, w["in_proj"], h, y_f32=self._buf("proj", T, w["in_proj"].shape[0], torch.float32), bias=w["in_bias"])
        out, at = self._buf("mixed", T, w["o"].shape[1], ctx.dtype), w["at"]
        if m.kind == "attention":
            self._window(ctx, i, m, proj, rows_at, out)
        elif m.kind == "delta":
            y = self._scan(ctx, i, proj, rows_at, m.heads, m.vdim_p)
            ops.gated_norm(ctx, y, proj[:, at["g"]:], w["norm"], out, m.vdim, m.heads, False, self.cfg.eps)
        else:
            a, r = m.left, m.right
            self._window(ctx, i, a, proj, rows_at, out, proj[:, at["gate"]:], m.left_scale)
            y = self._scan(ctx, i, proj, rows_at, r.heads, r.vdim_p)
            ops.gated_norm(ctx, y, proj[:, at["z"]:], w["norm"], out[:, a.heads * a.vdim_p:], r.vdim, r.norm_groups, True, self.cfg.eps,
                           m.right_scale)
        return ops.dense_linear(ctx, w["o"], out, y_f32=self._buf("delta", T, self.cfg.width_p, torch.float32), bias=w.get("o_bias"))

    # -- the layers -------------------------------------------------------------------------------------
    def _forward(self, tokens, rows_at, slots=None):
        """tokens (int32 device tensor) through every layer: final-normed rows [T, width padded]."""
        cfg, T = self.cfg, tokens.numel()
        ctx, D = self.pass_context(T), cfg.width
        x = self._buf("residual", T, D, torch.float32)
        h, last = self._buf("input", T, cfg.width_p, ctx.dtype), self._buf("normed", T, cfg.width_p, self.ctx.dtype)
        ops.embed_positions(ctx, self.w.embed, tokens, D, cfg.vocab, cfg.embed_scale, self.inv_freq, rows_at, x, h)
        for i, (m, ff) in enumerate(cfg.layers):
            w = self.w.layers[i]
            left = (ff is not None) + (cfg.side > 0)         # sublayers of this layer still to come

            def close(delta, weight, add):           # the end of a sublayer; behind the model's last one the final norm (in the head's type)
                if i + 1 == len(cfg.layers) and left == 0:
                    ops.rms_residual(self.ctx, x, D, delta, weight, add, self.w.final_norm, 1.0, last, cfg.eps)
                else:
                    ops.rms_residual(ctx, x, D, delta, weight, add, out=h, eps=cfg.eps)
            close(self._mix(ctx, i, h, rows_at), w["norm1"], 1.0)
            if ff is not None:
                left -= 1
                act = ops.dense_linear(ctx, w["gate_up"], h, y=self._buf("ff", T, w["down"].shape[1], ctx.dtype), activation=ops.LINEAR_SILU_PAIRS)
                close(ops.dense_linear(ctx, w["down"], act, y_f32=self._buf("delta", T, cfg.width_p, torch.float32)), w["norm2"], 1.0)
            if cfg.side:
                left -= 1
                g = ops.dense_linear(ctx, w["side_gate"], h, y=self._buf("side", T, w["side_proj"].shape[1], ctx.dtype),
                                     activation=ops.LINEAR_GELU_TANH, mul=w["side_embed"], mul_ids=tokens)
                close(ops.dense_linear(ctx, w["side_proj"], g, y_f32=self._buf("delta", T, cfg.width_p, torch.float32)), w["side_norm"], 0.0)
            if self.residual_hook is not None:
                self.residual_hook(i, x)
        return last

    def reset(self, sequence):
        """Forget what the sequence left: recurrent states start from zero (filter inputs before a sequence's start are not
        read, and ring rows are overwritten as they are used)."""
        for _, state in self.states.values():
            state[sequence].zero_()
