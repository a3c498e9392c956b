"""Trace replay: given token ids through a model's step function, logits out, nothing sampled.

Steps arrive on standard input, one JSON object a line::

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["a"]}

An entry's tokens continue its request from the cache that earlier steps left; ``want`` names the places among them
whose logits go to ``<out>/<step>.f32`` (little-endian fp32, ``[wanted, vocab]``, in the order asked; no file when
nothing is wanted).  ``end`` gives requests' caches back.  After every step ``done <step>`` is printed."""

from __future__ import annotations

import argparse
import json
import sys
from pathlib import Path


class Session:
    """Requests that are alive, each with a cache; caches of ended requests are used again."""

    def __init__(self, model, max_tokens: int) -> None:
        self.model = model
        self.max_len = min(max_tokens, model.context_length)
        self.live: dict = {}
        self.free: list = []

    def step(self, entries: list[dict], end: list[str]):
        """Runs the entries' tokens; returns the wanted logits ``[n, vocab]`` on the host, or None."""
        import torch

        wanted = []
        for entry in entries:
            tokens = entry["tokens"]
            if not tokens or min(tokens) < 0 or max(tokens) >= self.model.vocab_size:
                raise ValueError(f"request {entry['id']}: token ids must be in [0, {self.model.vocab_size})")
            if any(not 0 <= place < len(tokens) for place in entry["want"]):
                raise ValueError(f"request {entry['id']}: wanted places must be among the entry's tokens")
            cache = self.live.get(entry["id"])
            if cache is None:
                cache = self.free.pop() if self.free else self.model.new_cache(1, self.max_len)
                cache.reset()
                self.live[entry["id"]] = cache
            ids = torch.tensor([tokens], dtype=torch.long).to(self.model.token_embeddings.weight.device)
            logits = self.model(ids, cache, want=entry["want"])
            if entry["want"]:
                wanted.append(logits[0].float().cpu())
        for name in end:
            cache = self.live.pop(name, None)
            if cache is not None:
                self.free.append(cache)
        if wanted:
            return torch.cat(wanted, dim=0)
        torch.cuda.synchronize()
        return None


def main(argv: list[str] | None = None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.splitlines()[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", required=True, choices=("bfloat16", "float32"))
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, required=True, help="the most tokens live requests hold at any time")
    args = ap.parse_args(argv)

    from . import build

    build.ensure_dense_library()

    import torch

    from . import checkpoint

    torch.backends.cuda.matmul.allow_tf32 = False
    model = checkpoint.load_model(args.model, torch.device("cuda:0"), getattr(torch, args.dtype))
    session = Session(model, args.max_tokens)
    out = Path(args.out)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = session.step(step["entries"], step.get("end", []))
        if logits is not None:
            logits.contiguous().numpy().astype("<f4").tofile(out / f"{step['step']}.f32")
        print(f"done {step['step']}", flush=True)
    return 0
