"""Replay of a trace of given tokens: steps as JSON lines on standard input, logits as files.

A step is {"step": n, "entries": [{"id": .., "tokens": [..], "want": [..]}], "end": [..]}: the next tokens of each
request, the places among them whose logits are wanted, and the requests that are finished after it.  The logits of a
step go to OUT/<n>.f32, little-endian floats [wanted, vocab] in the order of the entries; every step is answered with a
line "done <n>"."""
import json
import os
import sys


def replay(decoder, lines, out_dir, write=None):
    import torch

    from .generate import Session
    session = Session(decoder)
    write = write or (lambda s: (sys.stdout.write(s + "\n"), sys.stdout.flush()))
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = []
        for e in step.get("entries", []):
            if not e["tokens"]:
                continue
            got = session.feed(e["id"], e["tokens"], e.get("want", []))
            if got is not None:
                rows.append(got.clone())
        if rows:
            logits = session.logits(torch.cat(rows) if len(rows) > 1 else rows[0])
            data = logits.cpu().numpy().astype("<f4", copy=False).tobytes()
            path = os.path.join(out_dir, "%s.f32" % step["step"])
            with open(path, "wb") as f:
                f.write(data)
        else:
            torch.cuda.synchronize()
        for request in step.get("end", []):
            if request in session:
                session.end(request)
        write("done %s" % step["step"])


def main(args):
    from .registry import open_model
    decoder = open_model(args.model, args.dtype, batch=args.slots, max_context=args.max_tokens)
    os.makedirs(args.out, exist_ok=True)
    replay(decoder, sys.stdin, args.out)
    return 0
