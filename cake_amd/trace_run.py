"""Replay given token ids through a model, step by step, and write logits (bin/trace_run).

Nothing is sampled: each step feeds every named sequence its next tokens as one batch through
the model's own step function and cache — the ones generation uses — and the logits of the
places asked for go to ``OUT/<step>.f32`` (little-endian f32, [wanted, vocab]).

Steps are JSON lines on standard input::

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

``end`` names the sequences finished after the step.  ``done <step>`` is printed after every
step.  The model class follows config.json (models/registry.py).
"""
from __future__ import annotations

import argparse
import json
import sys
from pathlib import Path

DTYPES = {"bfloat16": "bf16", "float32": "f32", "float16": "f16"}


class Replay:
    """Sequences by name over a model's step function."""

    def __init__(self, model):
        self.model = model
        self.seqs: dict[str, int] = {}

    def step(self, entries: list[dict], end: list[str]):
        """Logits [wanted, vocab] (None if nothing is wanted)."""
        import torch

        from .models.base import StepEntry
        batch = []
        for e in entries:
            if e["id"] not in self.seqs:
                self.seqs[e["id"]] = self.model.open_sequence()
            batch.append(StepEntry(self.seqs[e["id"]], [int(t) for t in e["tokens"]],
                                   [int(w) for w in e.get("want", [])]))
        out = self.model.step(batch) if batch else []
        for i in end:
            self.model.close_sequence(self.seqs.pop(i))
        got = [x for x in out if x.shape[0]]
        return torch.cat(got, 0).float().cpu() if got else None


def main(argv: list[str] | None = None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.splitlines()[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=sorted(DTYPES), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, default=4096,
                    help="most tokens that live sequences hold at any time")
    ap.add_argument("--device", type=int, default=0)
    a = ap.parse_args(argv)
    from . import build
    from .models.registry import family_of
    fam = family_of(a.model)
    build.ensure_text(fam.libs)
    import torch

    from .models.llama3.factory import parse_dtype
    if not torch.cuda.is_available():
        print("trace_run: no GPU", file=sys.stderr)
        return 1
    torch.cuda.set_device(a.device)
    model = fam.load_model(a.model, torch.device("cuda", a.device), parse_dtype(DTYPES[a.dtype]),
                           max(1, a.max_tokens))
    replay = Replay(model)
    out = Path(a.out)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = replay.step(s.get("entries", []), s.get("end", []))
        if logits is None:
            torch.cuda.synchronize()
        else:
            (out / f"{s['step']}.f32").write_bytes(logits.numpy().astype("<f4").tobytes())
        print(f"done {s['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
