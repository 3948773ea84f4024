"""Replays a trace of given token ids through a model, step by step, and writes logits (``bin/trace_run``).

Steps come on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

The entries of a step run as one batch on the continuous batcher (``ContinuousBatcher.feed``): requests named for
the first time take a slot, requests under "end" give theirs back after the step.  The logits at the wanted places
go to ``<out>/<step>.f32`` (little-endian fp32, [wanted, vocab], in the order of the entries), then ``done <step>`` is
printed.
"""

from __future__ import annotations

import argparse
import json
import os
import sys


class Replay:
    """Requests by name on a ``ContinuousBatcher``."""

    def __init__(self, model, slots: int = 1):
        from .batching import ContinuousBatcher

        self._new = lambda n: ContinuousBatcher(model, n)
        self.batcher = self._new(slots)
        self.slot: dict = {}

    def step(self, entries) -> list:
        """entries: (name, tokens) -> the logits (len(tokens), V) of each, in the same order."""
        fresh = sum(1 for name, _ in entries if name not in self.slot)
        if not self.slot and fresh and fresh != self.batcher.slots:
            # the batch a step opens decides how many rows the decode steps after it carry
            self.batcher = None  # the old caches go first
            self.batcher = self._new(fresh)
        out = self.batcher.feed([(self.slot.get(name), tokens) for name, tokens in entries])
        for (name, _), (b, _) in zip(entries, out):
            self.slot[name] = b
        return [logits for _, logits in out]

    def end(self, name) -> None:
        self.batcher.remove(self.slot.pop(name))


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay given token ids through a model and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder the logits are written to")
    ap.add_argument("--max-tokens", type=int, required=True, help="the most tokens that live requests hold at any time")
    args = ap.parse_args(argv)

    from . import build

    from .checkpoint import architecture_of, build_model, load_checkpoint

    build.ensure(architecture_of(args.model))

    import numpy as np
    import torch

    config, state = load_checkpoint(args.model, max_sequence_length=max(2, args.max_tokens))
    model = build_model(config, state, dtype=getattr(torch, args.dtype))
    del state
    replay = Replay(model)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = replay.step([(e["id"], e["tokens"]) for e in step["entries"]]) if step["entries"] else []
        rows = [lg[e["want"]] for e, lg in zip(step["entries"], logits) if e["want"]]
        if rows:
            data = torch.cat(rows).float().cpu().numpy().astype(np.dtype("<f4"))
            path = os.path.join(args.out, f"{step['step']}.f32")
            with open(path + ".part", "wb") as f:
                f.write(data.tobytes())
            os.replace(path + ".part", path)
        for name in step.get("end", ()):
            replay.end(name)
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
