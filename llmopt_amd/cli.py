"""Command line: python -m llmopt_amd {generate,replay,models} ...

    generate --model DIR --prompt 5,17,3 [--prompt ...] [--max-new-tokens N] [--temperature T --top-k K ...]
    replay   --model DIR --dtype bfloat16|float32 --out DIR [--max-tokens N]     (a trace on standard input)
    models                                                                       the known architectures

Token ids in, token ids out: tokenizers are not part of this package.
"""
from __future__ import annotations

import argparse
import os
import sys


def _tokens(text: str) -> list[int]:
    return [int(part) for part in text.replace(",", " ").split()]


def _parser() -> argparse.ArgumentParser:
    parser = argparse.ArgumentParser(prog="llmopt_amd")
    commands = parser.add_subparsers(dest="command", required=True)
    generate = commands.add_parser("generate", help="continue prompts of token ids")
    generate.add_argument("--model", required=True, help="a folder with config.json and its weights")
    generate.add_argument("--prompt", type=_tokens, action="append", required=True, help="token ids; may be repeated")
    generate.add_argument("--max-new-tokens", type=int, default=16)
    generate.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    generate.add_argument("--portion", type=int, default=2048, help="longest portion of a prompt per step")
    generate.add_argument("--max-context", type=int, default=32768)
    generate.add_argument("--slots", type=int, default=8, help="sequences that can be live at once")
    generate.add_argument("--temperature", type=float, default=0.0)
    generate.add_argument("--top-k", type=int, default=0)
    generate.add_argument("--top-p", type=float, default=1.0)
    generate.add_argument("--min-p", type=float, default=0.0)
    generate.add_argument("--seed", type=int, default=0)
    replay = commands.add_parser("replay", help="replay a trace from standard input and write logits")
    replay.add_argument("--model", required=True)
    replay.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    replay.add_argument("--out", required=True, help="folder for <step>.f32")
    replay.add_argument("--max-tokens", type=int, default=32768, help="the most tokens live requests hold together")
    commands.add_parser("models", help="list the known architectures")
    return parser


def main(argv=None) -> int:
    args = _parser().parse_args(argv)
    from . import model_registry
    if args.command == "models":
        print("\n".join(model_registry.architectures()))
        return 0
    if args.command == "replay":
        from . import trace_replay
        os.makedirs(args.out, exist_ok=True)
        model = model_registry.load_model(args.model, activations=args.dtype, max_context=max(1, args.max_tokens))
        trace_replay.replay(model, sys.stdin, args.out, trace_replay.answer_on_stdout)
        return 0
    from . import sampling
    from .engine import Engine
    model = model_registry.load_model(args.model, activations=args.dtype, slots=args.slots,
                                      max_context=args.max_context)
    params = sampling.Params.create(args.temperature, args.top_k, args.top_p, args.min_p, args.seed)
    for tokens in Engine(model, args.portion).generate(args.prompt, args.max_new_tokens, params):
        print(" ".join(str(token) for token in tokens))
    return 0


if __name__ == "__main__":
    sys.exit(main())
