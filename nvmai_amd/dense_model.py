"""What the dense models share: reading their configuration, laying weights out for the kernels, and the step driver
around their layers -- scratch rows, the context of short passes, slots and positions, logits.  A model supplies its
layers (`_forward`) and its states."""
import json
import os

import torch

from . import ops
from .decoder import StepDecoder
from .gturbo import ModelError
from .safetensors_file import SafetensorsFile

FEW_ROWS = 2        # passes whose products read 32-bit inputs at the price of 16-bit ones (dense_linear: bound by the weights)


def up(n, m):
    return (n + m - 1) // m * m


def need(d, where, *names):
    """The values of d at names; a model that lacks one is refused."""
    for n in names:
        if n not in d:
            raise ModelError("indexCorrupt", "config.json: %s has no %s" % (where, n))
    return [d[n] for n in names]


def blocks_of(t, dim, blocks, total=None):
    """Lay out `dim` of t anew: consecutive runs of `size` entries, each padded with zeros to `padded` (blocks =
    [(count, size, padded)]), the whole to `total`."""
    out_n = sum(c * p for c, _, p in blocks)
    total = out_n if total is None else total
    shape = list(t.shape)
    shape[dim] = total
    if total == t.shape[dim] and all(s == p for _, s, p in blocks):
        return t
    out = torch.zeros(shape, dtype=t.dtype, device=t.device)
    src = dst = 0
    for count, size, padded in blocks:
        lead = t.narrow(dim, src, count * size).unflatten(dim, (count, size))
        out.narrow(dim, dst, count * padded).unflatten(dim, (count, padded)).narrow(dim + 1, 0, size).copy_(lead)
        src, dst = src + count * size, dst + count * padded
    return out


def pad_columns(w):
    """A matrix with its k rounded up to what the products take."""
    return blocks_of(w, 1, [(1, w.shape[1], up(w.shape[1], 64))])


def open_directory(path, parse):
    """(configuration, tensor by name, shape by name) of a folder with config.json and model.safetensors."""
    with open(os.path.join(path, "config.json")) as f:
        cfg = parse(json.load(f))
    tensors = SafetensorsFile(os.path.join(path, "model.safetensors"))

    def shape(name):
        if name not in tensors:
            raise ModelError("indexCorrupt", "model.safetensors has no tensor %s" % name)
        return tensors.shape(name)
    return cfg, tensors.tensor, shape


def check_shapes(expected, shape):
    for name, want in expected.items():
        got = tuple(shape(name))
        if got != tuple(want):
            raise ModelError("indexCorrupt", "%s has shape %s, the configuration says %s" % (name, got, tuple(want)))


def bf16_reader(ctx, source):
    """name -> BF16 tensor on the context's device"""
    def t(name):
        v = source(name)
        if v.dtype != torch.bfloat16:
            raise ModelError("indexCorrupt", "%s must be BF16" % name)
        return v.to(ctx.device)
    return t


class DenseDecoder(StepDecoder):
    """Prompt portions and decode steps of a dense model for `batch` sequences (slots).  States and caches are allocated
    once; every call only enqueues kernels.  A model supplies _forward(tokens, rows_at, slots): int32 device tokens
    through every layer to final-normed rows [T, width padded]; weights.embed is the head."""
    long_f32 = ()               # names of 32-bit buffers that long passes use in a 16-bit context too

    def __init__(self, ctx, cfg, weights, batch=1, max_context=32768, max_chunk=2048):
        super().__init__(ctx, cfg, weights, batch, max_context)
        self.max_chunk = min(max_chunk, max_context)
        self.max_rows = max(self.max_chunk, batch)
        # Passes of a few rows are bound by the weights' bytes: their activations stay in 32 bits (a context of its own
        # over the same weights, states and caches); longer ones run in the context's type.
        self.few_ctx = ctx if ctx.act == ops.ACT_FP32 else ops.Context(ctx.device.index, ops.ACT_FP32)
        self.contexts = {ctx, self.few_ctx}
        self.slots = torch.arange(batch, dtype=torch.int32, device=ctx.device)
        self._buffers = {}
        self.residual_hook = None        # called with (layer index, residual rows) after every layer
        self.logits_f32 = torch.zeros((batch, cfg.vocab), dtype=torch.float32, device=ctx.device)

    def pass_context(self, rows):
        return self.few_ctx if rows <= FEW_ROWS else self.ctx

    def _buf(self, name, rows, cols, dtype):
        """Scratch rows.  Columns past a producer's own stay zero: a buffer's name goes with one width."""
        key = (name, cols, dtype)
        if key not in self._buffers:
            # buffers of passes in another type than the context's never see more than FEW_ROWS rows
            most = self.max_rows if dtype == self.ctx.dtype or name in self.long_f32 else FEW_ROWS
            self._buffers[key] = torch.zeros((most, cols), dtype=dtype, device=self.ctx.device)
        return self._buffers[key][:rows]

    def _prefill_chunk_rows(self, tokens, b, start):
        return self._forward(tokens, ops.row_map(b, start))

    def forward_hidden(self, position):
        """One token (self.tokens) of every sequence at `position` (None: each at its own, self.positions)."""
        if position is not None:
            self.positions.fill_(position)
        rows_at = ops.row_map(slots=self.slots, positions=self.positions, most=self.max_context - 1 if position is None else position)
        self.normed = self._forward(self.tokens, rows_at, self.slots)
        return self.normed

    def decode_rows(self, sequences, positions, tokens):
        if max(positions) >= self.max_context:
            raise ValueError("position %d exceeds the context (%d)" % (max(positions), self.max_context))
        ids = torch.tensor([tokens, sequences, positions], dtype=torch.int32).to(self.ctx.device)
        if len(sequences) == 1:
            return self._forward(ids[0], ops.row_map(sequences[0], positions[0]))
        return self._forward(ids[0], ops.row_map(slots=ids[1], positions=ids[2], most=max(positions)), ids[1])

    # -- logits -----------------------------------------------------------------------------------------
    def head_rows(self, normed):
        """(activations, 32-bit) logits of any number of final-normed rows, before the cap."""
        n = normed.shape[0]
        y32 = torch.empty((n, self.cfg.vocab), dtype=torch.float32, device=self.ctx.device)
        if self.ctx.act == ops.ACT_FP32:
            ops.dense_linear(self.ctx, self.w.embed, normed, y_f32=y32)
            return y32, y32
        y = torch.empty((n, self.cfg.vocab), dtype=self.ctx.dtype, device=self.ctx.device)
        ops.dense_linear(self.ctx, self.w.embed, normed, y=y, y_f32=y32)
        return y, y32

    def head(self):
        """Logits of the rows forward_hidden left: activations in self.logits, 32-bit in self.logits_f32."""
        ops.dense_linear(self.ctx, self.w.embed, self.normed, y=self.logits, y_f32=self.logits_f32)
        return self.logits

    def greedy(self):
        """Greedy tokens of self.logits_f32 in self.next_tokens (a cap of the logits keeps their order)."""
        return ops.argmax_rows(self.ctx, self.logits_f32, out=self.next_tokens)
