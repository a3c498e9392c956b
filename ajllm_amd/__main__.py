"""Command line: ``python -m ajllm_amd generate --model DIR --tokens 1,2,3 --max-new-tokens N``.

Continues a prompt of token ids with the model a folder holds (``config.json``, ``model.safetensors``) and prints the
new ids, one line per prompt.  ``--tokens`` may be given several times with prompts of equal length: they are decoded as
one batch."""

from __future__ import annotations

import argparse
import sys


def main(argv: list[str] | None = None) -> int:
    ap = argparse.ArgumentParser(prog="ajllm_amd", description="Token generation on a ROCm device.")
    commands = ap.add_subparsers(dest="command", required=True)
    gen = commands.add_parser("generate", help="continue prompts of token ids")
    gen.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    gen.add_argument("--dtype", default="bfloat16", choices=("bfloat16", "float32"))
    gen.add_argument("--tokens", required=True, action="append", help="a prompt: ids separated by commas (repeat for a batch)")
    gen.add_argument("--max-new-tokens", type=int, default=32)
    gen.add_argument("--temperature", type=float, default=0.0, help="0: the most probable token")
    gen.add_argument("--top-p", type=float, default=None)
    gen.add_argument("--seed", type=int, default=0)
    gen.add_argument("--eos", type=int, default=None, help="stop once every prompt has produced this id")
    args = ap.parse_args(argv)
    prompts = [[int(t) for t in text.split(",")] for text in args.tokens]
    if len({len(p) for p in prompts}) != 1:
        ap.error("the prompts of a batch must have equal length")

    import torch

    from . import checkpoint, decoding

    model = checkpoint.load_model(args.model, torch.device("cuda:0"), getattr(torch, args.dtype))
    if any(not 0 <= t < model.vocab_size for p in prompts for t in p):
        ap.error(f"token ids must be in [0, {model.vocab_size})")
    decoder = decoding.decoder_for(model)(model, len(prompts), len(prompts[0]) + args.max_new_tokens)
    if args.temperature > 0:
        decoder.set_sampling(args.temperature, args.top_p, args.seed)
    decoder.prefill(torch.tensor(prompts))
    for row in decoder.generate(args.max_new_tokens, args.eos).tolist():
        print(",".join(str(t) for t in row))
    return 0


if __name__ == "__main__":
    sys.exit(main())
