"""Replay of recorded token ids through a model (bin/trace_run), for comparing logits between builds, dtypes and ways of
cutting a sequence.

Steps come as JSON lines on standard input: `step` (a number), `entries` (per request: `id`, the next `tokens`, and `want`,
indices into them) and `end` (ids that are done).  For example

    {"step": 7, "entries": [{"id": "chat-1", "tokens": [101, 9], "want": [1]}], "end": ["chat-1"]}

A request's tokens continue from the cache its earlier steps left.  Wanted logits go to <out>/<step>.f32 as rows of
little-endian float32, entry by entry; each finished step is acknowledged by a line "done <step>".  An ended request's cache
memory is used again by later requests.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, List, Optional

import torch

DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}


class Replayer:
    """A model and the caches of the requests that are running."""

    def __init__(self, model, max_tokens: int):
        self.model, self.max_tokens = model, max_tokens
        self.live: Dict[str, tuple] = {}
        self.free: List[tuple] = []

    @torch.no_grad()
    def feed(self, request: str, tokens: List[int], want: List[int]) -> Optional[torch.Tensor]:
        """-> float32 logits [len(want), vocab], None if nothing is wanted."""
        dev, vocab = self.model.device, self.model.config.vocab_size
        if not all(0 <= t < vocab for t in tokens) or not all(0 <= w < len(tokens) for w in want):
            raise ValueError("request %s: a token is not in the vocabulary, or a wanted place not among the tokens" % request)
        past = self.live.get(request)
        if past is None:
            past = self.free.pop() if self.free else self.model.new_cache(1, max(self.max_tokens, len(tokens)))
        ids = torch.tensor([tokens], dtype=torch.long, device=dev)
        places = torch.tensor(want if want else [len(tokens) - 1], dtype=torch.long, device=dev)
        out = self.model(input_ids=ids, past_key_values=past, logit_positions=places)
        self.live[request] = out.past_key_values
        return out.logits[0].float() if want else None

    def end(self, request: str) -> None:
        past = self.live.pop(request, None)
        if past is not None:
            self.free.append(self.model.reset_cache(past))


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay token ids through a model and write logits.")
    ap.add_argument("--model", required=True, help="checkpoint directory (config.json, safetensors)")
    ap.add_argument("--dtype", choices=sorted(DTYPES), default="bfloat16")
    ap.add_argument("--out", required=True, help="directory for <step>.f32")
    ap.add_argument("--max-tokens", type=int, default=1024, help="most tokens the running requests hold at any time")
    args = ap.parse_args(argv)

    from . import build
    from .checkpoint import load_pretrained
    from .registry import family_of
    with open(os.path.join(args.model, "config.json")) as f:
        family = family_of(json.load(f))
    if family.polar_cache:
        print("trace_run: %s models run in half precision on whole prompts only" % family.name, file=sys.stderr)
        return 2
    build.ensure(family.libraries, verbose=False)
    torch.backends.cuda.matmul.allow_tf32 = False
    torch.backends.cuda.matmul.allow_bf16_reduced_precision_reduction = False
    model = load_pretrained(args.model, DTYPES[args.dtype], "cuda:0")
    replay = Replayer(model, args.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = [replay.feed(e["id"], e["tokens"], e["want"]) for e in step["entries"] if e["tokens"]]
        rows = [r for r in rows if r is not None]
        if rows:
            with open(os.path.join(args.out, "%d.f32" % step["step"]), "wb") as f:
                f.write(torch.cat(rows).cpu().numpy().astype("<f4").tobytes())
        for request in step["end"]:
            replay.end(request)
        print("done %d" % step["step"], flush=True)
    return 0
