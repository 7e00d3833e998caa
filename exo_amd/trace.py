"""Replay a trace of token ids through a model, step by step, and write the logits asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N  < steps

Standard input holds one JSON object per line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

The entries of a step are one batch of the model's own step function; ``want`` lists places among
an entry's tokens.  DIR/<step>.f32 receives their logits (little-endian float32 [wanted, vocab]) in
entry order.  ``end`` names requests that are finished after the step: their pages and row are
given back.  After each step the line ``done <step>`` is printed.  Nothing is sampled.
"""

from __future__ import annotations

import argparse
import json
import sys
from pathlib import Path

ROWS = 4  # live requests


def ensure_built() -> None:
    """Compile the kernel library if this checkout has none."""
    from . import native
    if not native.LIB_PATH.exists():
        from .build import build
        build(verbose=False)


class Replay:
    """Requests of a trace on the rows of one cache."""

    def __init__(self, model, max_tokens: int, rows: int = ROWS):
        from .paged_cache import PAGE, pages_for
        self.model = model
        n = max(1, pages_for(max_tokens)) * PAGE
        self.cache = model.make_cache(rows, n, pool_tokens=n)
        self.free = list(range(rows - 1, -1, -1))
        self.row: dict[str, int] = {}

    def step(self, entries: list[dict], end: list[str]):
        """Logits of the wanted places as a float32 array, or None."""
        batch = []
        for e in entries:
            if e["id"] not in self.row:
                if not self.free:
                    raise RuntimeError(f"more than {self.cache.batch} live requests")
                self.row[e["id"]] = self.free.pop()
            if e["tokens"]:
                batch.append((self.row[e["id"]], e["tokens"], e.get("want") or []))
        out = self.model.step(self.cache, batch) if batch else None
        logits = None if out is None else out.float().cpu().numpy()
        for name in end:
            if name in self.row:
                self.cache.release(self.row[name])
                self.free.append(self.row.pop(name))
        return logits


def main(argv: list[str] | None = None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n\n")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for the <step>.f32 files")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    a = ap.parse_args(argv)
    ensure_built()
    import torch

    from .registry import load_model
    model = load_model(a.model, dtype=getattr(torch, a.dtype))
    if not getattr(model, "mixed_steps", False):
        raise ValueError(f"{model.cfg.model_type}: no step function that mixes portions of prompts and decoded tokens")
    replay, out = Replay(model, a.max_tokens), Path(a.out)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = replay.step(s.get("entries") or [], s.get("end") or [])
        if logits is not None:
            (out / f"{s['step']}.f32").write_bytes(logits.astype("<f4").tobytes())
        else:
            torch.cuda.synchronize()
        print(f"done {s['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
