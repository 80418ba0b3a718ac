"""Command line of the framework.  Parsing needs no library; the commands load it."""
import argparse
import json
import sys


def parser():
    ap = argparse.ArgumentParser(prog="nvmai_amd")
    sub = ap.add_subparsers(dest="command", required=True)
    r = sub.add_parser("replay", help="feed given tokens step by step (JSON lines on stdin) and write logits")
    g = sub.add_parser("generate", help="continue prompts of token ids")
    for p in (r, g):
        p.add_argument("--model", required=True, help="model directory")
        p.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float16", "float32"])
    r.add_argument("--out", required=True, help="folder for <step>.f32")
    r.add_argument("--max-tokens", type=int, default=32768, help="most tokens of live requests: sizes the cache")
    r.add_argument("--slots", type=int, default=1, help="requests that may be open at once")
    g.add_argument("--prompt", action="append", required=True, metavar="IDS", help="token ids with commas between them; repeatable")
    g.add_argument("--max-new", type=int, default=16)
    g.add_argument("--max-context", type=int, default=32768)
    g.add_argument("--batch", type=int, default=1, help="requests decoded together")
    g.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    g.add_argument("--top-k", type=int, default=None)
    g.add_argument("--top-p", type=float, default=None)
    g.add_argument("--repetition-penalty", type=float, default=1.0)
    g.add_argument("--seed", type=int, default=None)
    g.add_argument("--stop", default="", metavar="IDS", help="token ids that end a request")
    return ap


def _ids(text):
    return [int(t) for t in text.split(",") if t.strip()]


def generate(args):
    from . import ops
    from .generate import Generator
    from .registry import open_model
    decoder = open_model(args.model, args.dtype, batch=args.batch, max_context=args.max_context)
    config = ops.GenerationConfig(args.temperature, args.top_k, args.top_p, args.repetition_penalty, args.seed)
    prompts = [_ids(p) for p in args.prompt]
    for new in Generator(decoder, _ids(args.stop)).generate(prompts, args.max_new, config):
        print(json.dumps(new), flush=True)
    return 0


def main(argv=None):
    args = parser().parse_args(argv)
    if args.command == "replay":
        from .replay import main as run
        return run(args)
    return generate(args)


if __name__ == "__main__":
    sys.exit(main())
