"""Sessions over a step driver: requests are given slots, fed in portions of any size, decoded together, and give their
slot back.  `Session` is what a trace replay and the generator share; `Generator` is the text-free generation loop
(token ids in, token ids out) with the sampler."""
import torch

from . import ops


class Session:
    """Requests on a step driver's slots.  A request is one sequence: what it has been fed is in the driver's caches and
    states, and only its new tokens are run."""

    def __init__(self, decoder):
        self.decoder = decoder
        self._free = list(range(decoder.batch))
        self._slot, self._length = {}, {}

    def __contains__(self, request):
        return request in self._slot

    @property
    def free_slots(self):
        return len(self._free)

    def length(self, request):
        return self._length[request]

    def open(self, request):
        if request in self._slot:
            raise ValueError("request %r is open" % (request,))
        if not self._free:
            raise RuntimeError("no free slot for request %r" % (request,))
        slot = self._free.pop(0)
        self.decoder.reset(slot)
        self._slot[request], self._length[request] = slot, 0

    def end(self, request):
        self._free.append(self._slot.pop(request))
        del self._length[request]

    def feed(self, request, tokens, want=None):
        """The next tokens of a request; final-normed rows at the places `want` (None: the last; () : none)."""
        if request not in self._slot:
            self.open(request)
        slot, at = self._slot[request], self._length[request]
        if len(tokens) == 1 and at > 0:
            rows = self.decoder.decode_rows([slot], [at], list(tokens))
            rows = rows if want is None or len(want) == 1 else (None if len(want) == 0 else rows.repeat(len(want), 1))
        else:
            ids = torch.tensor(list(tokens), dtype=torch.int32).to(self.decoder.ctx.device)
            rows = self.decoder.prefill_rows(ids, slot, at, want)
        self._length[request] = at + len(tokens)
        return rows

    def decode(self, requests, tokens):
        """One more token of each of several open requests: final-normed rows in their order."""
        slots, at = [self._slot[r] for r in requests], [self._length[r] for r in requests]
        rows = self.decoder.decode_rows(slots, at, list(tokens))
        for r in requests:
            self._length[r] += 1
        return rows

    def logits(self, rows):
        """32-bit logits of final-normed rows."""
        return self.decoder.logits_rows(rows)


class Generator:
    """Continuous generation: waiting prompts take free slots as they come, running requests decode together."""

    def __init__(self, decoder, stop_tokens=()):
        self.decoder, self.stop = decoder, frozenset(stop_tokens)

    def _next(self, rows, histories, positions, config, samplers):
        y, y32 = self.decoder.head_rows(rows)
        if config.temperature == 0.0 and config.repetition_penalty == 1.0 and y32 is not None:
            return ops.argmax_rows(self.decoder.ctx, y32).tolist()
        out = [s.sample(y[j], histories[j], config, positions[j])[0] for j, s in enumerate(samplers)]
        return torch.cat(out).tolist()

    def generate(self, prompts, max_new_tokens, config=None, on_token=None):
        """prompts: lists of token ids.  Returns the new ids of each (a stop token ends a request and is kept).
        config: ops.GenerationConfig (default: greedy); on_token(index, token) as they come."""
        config = config or ops.GenerationConfig(temperature=0.0, top_k=None, top_p=None)
        if any(len(p) == 0 for p in prompts):
            raise ValueError("a prompt needs at least one token")
        limit = self.decoder.max_context
        for p in prompts:
            if len(p) + max_new_tokens - 1 > limit:
                raise ValueError("prompt of %d tokens and %d new ones exceed the context (%d)" % (len(p), max_new_tokens, limit))
        new = [[] for _ in prompts]
        if max_new_tokens < 1:
            return new
        session = Session(self.decoder)
        sampler = lambda: ops.Sampler(self.decoder.ctx, self.decoder.cfg.vocab, self.decoder.cfg.logit_softcap)
        samplers = {}
        waiting, running = list(range(len(prompts))), []

        def took(i, token):
            new[i].append(token)
            if on_token is not None:
                on_token(i, token)
            if len(new[i]) >= max_new_tokens or token in self.stop:
                session.end(i)
                if i in running:
                    running.remove(i)
            elif i not in running:
                running.append(i)

        while waiting or running:
            while waiting and session.free_slots:
                i = waiting.pop(0)
                samplers[i] = sampler()
                rows = session.feed(i, prompts[i])
                took(i, self._next(rows, [prompts[i]], [len(prompts[i])], config, [samplers[i]])[0])
            if running:
                ids = list(running)
                rows = session.decode(ids, [new[i][-1] for i in ids])
                tokens = self._next(rows, [list(prompts[i]) + new[i] for i in ids], [session.length(i) for i in ids], config,
                                    [samplers[i] for i in ids])
                for i, token in zip(ids, tokens):
                    took(i, token)
        return new
