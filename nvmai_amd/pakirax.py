"""Pakirax: a decoder-only language model of gated-linear-attention and windowed latent-attention layers, with a norm
before and after every sublayer.  Configuration, weights and step driver; what its step driver shares with the other
dense models is in dense_model.py.

A layer is  x <- x + m norm1b(mixer(norm1 x))  and, when it has a feed-forward,  x <- x + m norm2b(ff(norm2 x));  the
residual x is 32-bit, the norms are layer norms with weight and bias, the logits are the embedding table times the
final-normed row.  Every size and constant comes from config.json or from a tensor's shape, layer by layer.

Weights are laid out for one launch per projection group (q, k, v, gate and the decay's first matrix of a GLA layer; both
down projections and the output gate of a latent-attention layer are rows of one matrix each) and padded with zeros so
that the kernels see multiples of 16 (heads) and 64 (the k of a product); real counts go with them where a norm needs
them."""
import torch

from . import ops
from .dense_model import DenseDecoder, bf16_reader, blocks_of, check_shapes, need, open_directory, pad_columns, up
from .gturbo import ModelError


class GlaLayer:
    kind = "gla"

    def __init__(self, m, where):
        self.heads, self.dim, self.vdim, self.tau = need(m, where, "heads", "dim", "vdim", "tau")
        self.dim_p, self.vdim_p = up(self.dim, 16), up(self.vdim, 16)

    def shapes(self, width, rank):
        kd, vd = self.heads * self.dim, self.heads * self.vdim
        return {"q": (kd, width), "k": (kd, width), "v": (vd, width), "g": (vd, width), "o": (width, vd), "norm": (self.vdim,),
                "a1": (rank, width), "a2": (kd, rank), "a2.b": (kd,)}


class LatentLayer:
    kind = "latent_attention"

    def __init__(self, m, where):
        (self.heads, self.dim, self.rot_dim, self.vdim, self.kv_rank, self.q_rank, self.scale) = \
            need(m, where, "heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank", "scale")
        rot, mask = m.get("rot"), m.get("mask")
        self.rot_base, self.rot_dims = (float(rot["base"]), int(rot["dims"])) if rot else (1.0, 0)
        self.window = int(mask["size"]) if mask else 0
        if self.rot_dims > self.rot_dim or self.rot_dims % 2 or (mask and self.window < 1):
            raise ModelError("indexCorrupt", "config.json: %s: rot or mask out of range" % where)
        self.dim_p, self.rot_p, self.vdim_p, self.rank_p = up(self.dim, 16), up(self.rot_dim, 16), up(self.vdim, 16), up(self.kv_rank, 64)

    def shapes(self, width, rank):
        H = self.heads
        return {"dq": (self.q_rank, width), "dq.norm": (self.q_rank,), "uq": (H * (self.dim + self.rot_dim), self.q_rank),
                "dkv": (self.kv_rank + self.rot_dim, width), "dkv.norm": (self.kv_rank,), "uk": (H * self.dim, self.kv_rank),
                "uv": (H * self.vdim, self.kv_rank), "g": (H, width), "o": (width, H * self.vdim)}


MIXERS = {"gla": GlaLayer, "latent_attention": LatentLayer}


class PakiraxConfig:
    """config.json, checked.  layers: one (mixer, ff or None) per layer."""

    def __init__(self, config):
        self.vocab, self.width, self.residual_mult, norm, layers = \
            need(config, "the model", "vocab", "width", "residual_mult", "norm", "layers")
        self.eps, = need(norm, "norm", "eps")
        self.hidden = self.width
        self.width_p = up(self.width, 64)
        self.logit_softcap = 0.0
        self.layers = []
        for i, e in enumerate(layers):
            kind, mixer = need(e, "layer %d" % i, "type", "mixer")
            if kind not in MIXERS:
                raise ModelError("unsupportedArch", "layer %d: mixer %s" % (i, kind))
            ff = None
            if e.get("mlp") is not None:
                mlp_kind, ff = need(e["mlp"], "layer %d's mlp" % i, "kind", "ff")
                if mlp_kind != "dense":
                    raise ModelError("unsupportedArch", "layer %d: feed-forward %s" % (i, mlp_kind))
            self.layers.append((MIXERS[kind](mixer, "layer %d" % i), ff))

    def tensor_shapes(self, decay_rank):
        """Name -> shape of every tensor; decay_rank: layer index -> rows of that layer's a1."""
        W = self.width
        out = {"embed": (self.vocab, W), "final.norm": (W,), "final.norm.b": (W,)}
        for i, (m, ff) in enumerate(self.layers):
            for n in ("norm1", "norm1b") + (("norm2", "norm2b") if ff is not None else ()):
                out["l%d.%s" % (i, n)] = out["l%d.%s.b" % (i, n)] = (W,)
            for n, s in m.shapes(W, decay_rank(i)).items():
                out["l%d.mix.%s" % (i, n)] = s
            if ff is not None:
                out["l%d.mlp.up" % i], out["l%d.mlp.down" % i] = (ff, W), (W, ff)
        return out

    def matrix_elements(self, decay_rank=16):
        """Elements of every matrix a token is multiplied by, the logits' included."""
        shapes = self.tensor_shapes(lambda i: decay_rank)
        return sum(s[0] * s[1] for s in shapes.values() if len(s) == 2)

    def bytes_per_token(self, batch=1, context=32768, act_bytes=2):
        """Algorithmic HBM bytes of one decode step divided by the batch: every matrix once, recurrent states read and
        written, the cached rows the windows reach."""
        own = 0
        for m, _ in self.layers:
            if m.kind == "gla":
                own += 2 * 4 * m.heads * m.dim * m.vdim
            else:
                own += act_bytes * (min(context, m.window) if m.window else context) * (m.kv_rank + m.rot_dim)
        return 2 * self.matrix_elements() / batch + own

    def prefill_flops(self, tokens):
        """Useful flops of a prompt of `tokens`: 2 per matrix element and token (the logits of one token), the pairs
        inside the windows, the recurrences' two products."""
        total = 2.0 * tokens * (self.matrix_elements() - self.vocab * self.width) + 2.0 * self.vocab * self.width
        for m, _ in self.layers:
            if m.kind == "gla":
                total += 4.0 * tokens * m.heads * m.dim * m.vdim
            else:
                w = min(m.window or tokens, tokens)
                total += 2.0 * m.heads * (m.dim + m.rot_dim + m.vdim) * (w * (w + 1) / 2 + (tokens - w) * w)
        return total


class PakiraxWeights:
    """Device tensors of a model, padded and grouped.  source(name) -> BF16 tensor; shape(name) -> its shape."""

    def __init__(self, ctx, cfg, source, shape):
        self.ctx, self.cfg = ctx, cfg
        rank = lambda i: shape("l%d.mix.a1" % i)[0] if cfg.layers[i][0].kind == "gla" else 0
        check_shapes(cfg.tensor_shapes(rank), shape)
        t, cols = bf16_reader(ctx, source), pad_columns
        norm = lambda n: (t(n).contiguous(), t(n + ".b").contiguous())
        self.embed = cols(t("embed")).contiguous()
        self.final_norm = norm("final.norm")
        self.layers = []
        for i, (m, ff) in enumerate(cfg.layers):
            p, x = "l%d." % i, "l%d.mix." % i
            w = dict(norm1=norm(p + "norm1"), norm1b=norm(p + "norm1b"))
            H = m.heads
            if m.kind == "gla":
                r, rp = rank(i), up(rank(i), 16)
                kd, vd = H * m.dim_p, H * m.vdim_p
                rows = [blocks_of(t(x + n), 0, [(H, m.dim, m.dim_p)]) for n in ("q", "k")] + \
                       [blocks_of(t(x + n), 0, [(H, m.vdim, m.vdim_p)]) for n in ("v", "g")] + [blocks_of(t(x + "a1"), 0, [(1, r, rp)])]
                w["in_proj"] = cols(torch.cat(rows)).contiguous()
                w["at"] = dict(q=0, k=kd, v=2 * kd, g=2 * kd + vd, a1=2 * kd + 2 * vd)
                w["a2"] = blocks_of(blocks_of(t(x + "a2"), 0, [(H, m.dim, m.dim_p)]), 1, [(1, r, rp)]).contiguous()
                w["a2_bias"] = blocks_of(t(x + "a2.b"), 0, [(H, m.dim, m.dim_p)]).contiguous()
                w["norm"] = blocks_of(t(x + "norm"), 0, [(1, m.vdim, m.vdim_p)]).contiguous()
                w["rank"] = rp
            else:
                qp, gp = up(m.q_rank, 16), up(H, 16)
                rows = [blocks_of(t(x + "dq"), 0, [(1, m.q_rank, qp)]),
                        blocks_of(t(x + "dkv"), 0, [(1, m.kv_rank, m.rank_p), (1, m.rot_dim, m.rot_p)]),
                        blocks_of(t(x + "g"), 0, [(1, H, gp)])]
                w["in_proj"] = cols(torch.cat(rows)).contiguous()
                w["at"] = dict(q=0, kv=qp, rope=qp + m.rank_p, g=qp + m.rank_p + m.rot_p)
                uq = t(x + "uq").unflatten(0, (H, m.dim + m.rot_dim))
                uq = torch.cat([blocks_of(uq[:, :m.dim], 1, [(1, m.dim, m.dim_p)]),
                                blocks_of(uq[:, m.dim:], 1, [(1, m.rot_dim, m.rot_p)])], 1).flatten(0, 1)
                w["uq"] = cols(uq).contiguous()
                w["uk"] = cols(blocks_of(t(x + "uk"), 0, [(H, m.dim, m.dim_p)])).contiguous()
                w["uv"] = cols(blocks_of(t(x + "uv"), 0, [(H, m.vdim, m.vdim_p)])).contiguous()
                w["q_norm"] = blocks_of(t(x + "dq.norm"), 0, [(1, m.q_rank, qp)]).contiguous()
                w["kv_norm"] = blocks_of(t(x + "dkv.norm"), 0, [(1, m.kv_rank, m.rank_p)]).contiguous()
            w["o"] = blocks_of(t(x + "o"), 1, [(H, m.vdim, m.vdim_p)], up(H * m.vdim_p, 64)).contiguous()
            if ff is not None:
                w.update(norm2=norm(p + "norm2"), norm2b=norm(p + "norm2b"), up=cols(t(p + "mlp.up")).contiguous(),
                         down=cols(t(p + "mlp.down")).contiguous())
            self.layers.append(w)

    @classmethod
    def from_directory(cls, ctx, path):
        """(config, weights) of a folder with config.json and model.safetensors."""
        cfg, tensor, shape = open_directory(path, PakiraxConfig)
        return cfg, cls(ctx, cfg, tensor, shape)

    @classmethod
    def random(cls, ctx, cfg, seed=1234, decay_rank=16):
        """Random-init weights on the device, scaled so that activations stay of order one."""
        gen = torch.Generator(device=ctx.device).manual_seed(seed)
        shapes = cfg.tensor_shapes(lambda i: decay_rank)

        def source(name):
            s = shapes[name]
            v = torch.empty(s, dtype=torch.float32, device=ctx.device)
            if len(s) == 1:
                v.normal_(0.0, 0.1, generator=gen)
                if not name.endswith(".b"):
                    v += 1.0
                elif name.endswith("a2.b"):
                    v += 2.0
            else:
                v.normal_(0.0, s[1] ** -0.5, generator=gen)
            return v.to(torch.bfloat16)
        return cls(ctx, cfg, source, lambda n: shapes[n])


class PakiraxDecoder(DenseDecoder):
    """Prompt portions and decode steps of a Pakirax model.  A ring holds the layer's window beside one portion of
    max_chunk tokens, so a layer's cache does not grow with the context."""
    long_f32 = ("residual", "delta", "gla_proj")

    def __init__(self, ctx, cfg, weights, batch=1, max_context=32768, max_chunk=2048):
        super().__init__(ctx, cfg, weights, batch, max_context, max_chunk)
        self.mixers, self.states, self.caches = {}, {}, {}
        for i, (m, _) in enumerate(cfg.layers):
            for c in self.contexts:
                if m.kind == "gla":
                    op = ops.GLA(c, m.heads, m.dim_p, m.vdim_p, weights.layers[i]["rank"], m.tau, cfg.eps, m.dim, m.vdim)
                else:
                    op = ops.LatentAttention(c, m.heads, m.dim_p, m.rot_p, m.vdim_p, m.rank_p, m.kv_rank, m.scale, m.window,
                                             m.rot_dims, m.rot_base, cfg.eps)
                self.mixers[i, c] = op
            if m.kind == "gla":
                self.states[i] = op.new_state(batch)
            else:
                capacity = min(max_context, m.window + self.max_chunk - 1) if m.window else max_context
                self.caches[i] = ops.LatentCache(ctx, batch, capacity, m.rank_p, m.rot_p)

    # -- mixers: normed rows in, the sublayer's output as 32-bit rows ---------------------------------------
    def _gla(self, ctx, i, h, rows_at, T, slots):
        m, w, op = self.cfg.layers[i][0], self.w.layers[i], self.mixers[i, ctx]
        proj = ops.dense_linear(ctx, w["in_proj"], h, y_f32=self._buf("gla_proj", T, w["in_proj"].shape[0], torch.float32))
        part = lambda n: proj[:, w["at"][n]:]
        out = self._buf("gla_out%d" % (m.heads * m.vdim_p), T, w["o"].shape[1], ctx.dtype)
        batch, rows = (1, T) if slots is None else (T, 1)
        op.encode(part("q"), part("k"), part("v"), part("g"), part("a1"), w["a2"], w["a2_bias"], w["norm"], self.states[i], out,
                  rows, batch, rows_at.slot, slots)
        return ops.dense_linear(ctx, w["o"], out, y_f32=self._buf("delta", T, self.cfg.width_p, torch.float32))

    def _latent_attention(self, ctx, i, h, rows_at, T, slots):
        m, w, op = self.cfg.layers[i][0], self.w.layers[i], self.mixers[i, ctx]
        at, dt = w["at"], ctx.dtype
        proj = ops.dense_linear(ctx, w["in_proj"], h, y=self._buf("latent_proj", T, w["in_proj"].shape[0], dt))
        cq = self._buf("cq%d" % m.q_rank, T, w["uq"].shape[1], dt)
        op.encode_epilogue(proj, at["q"], m.q_rank, w["q_norm"], at["kv"], at["rope"], w["kv_norm"], cq, self.caches[i], rows_at)
        q = ops.dense_linear(ctx, w["uq"], cq, y=self._buf("latent_q", T, w["uq"].shape[0], dt))
        out = self._buf("latent_out%d" % (m.heads * m.vdim_p), T, w["o"].shape[1], dt)
        op.encode(q, proj[:, at["g"]:], w["uk"], w["uv"], self.caches[i], rows_at, out)
        return ops.dense_linear(ctx, w["o"], out, y_f32=self._buf("delta", T, self.cfg.width_p, torch.float32))

    # -- the layers -------------------------------------------------------------------------------------
    def _forward(self, tokens, rows_at, slots=None):
        """tokens (int32 device tensor) through every layer: final-normed rows [T, width padded]."""
        cfg, T = self.cfg, tokens.numel()
        ctx = self.pass_context(T)
        D, mult = cfg.width, cfg.residual_mult
        x = self._buf("residual", T, D, torch.float32)
        h, last = self._buf("normed", T, cfg.width_p, ctx.dtype), self._buf("normed", T, cfg.width_p, self.ctx.dtype)
        ops.embed_rows(ctx, self.w.embed, tokens, D, cfg.vocab, x)

        def close(delta, post, layer):           # the end of a sublayer and the norm of layer `layer` (the final one: the head's type)
            if layer < len(cfg.layers):
                ops.norm_residual(ctx, x, D, delta, post, mult, self.w.layers[layer]["norm1"], h, cfg.eps)
            else:
                ops.norm_residual(self.ctx, x, D, delta, post, mult, self.w.final_norm, last, cfg.eps)
        close(None, None, 0)
        for i, (m, ff) in enumerate(cfg.layers):
            w = self.w.layers[i]
            delta = (self._gla if m.kind == "gla" else self._latent_attention)(ctx, i, h, rows_at, T, slots)
            if ff is None:
                close(delta, w["norm1b"], i + 1)
            else:
                ops.norm_residual(ctx, x, D, delta, w["norm1b"], mult, w["norm2"], h, cfg.eps)
                act = ops.dense_linear(ctx, w["up"], h, y=self._buf("ff%d" % ff, T, w["down"].shape[1], ctx.dtype), activation=ops.LINEAR_GELU_ERF)
                delta = ops.dense_linear(ctx, w["down"], act, y_f32=self._buf("delta", T, cfg.width_p, torch.float32))
                close(delta, w["norm2b"], i + 1)
            if self.residual_hook is not None:
                self.residual_hook(i, x)
        return last

    def reset(self, sequence):
        """Forget what the sequence left: recurrent states start from zero (ring rows are overwritten as they are used)."""
        for state in self.states.values():
            state[sequence].zero_()
