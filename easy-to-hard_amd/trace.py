"""Replay a trace of requests through a model: given token ids in, logits out, nothing sampled.

The trace is a sequence of JSON lines, one step each:
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
Each entry brings a request's next tokens; `want` lists the places among them whose logits are stored as little-endian
float32 rows in <out>/<step>.f32, entry by entry.  `end` names the requests that are finished.  After every step a line
"done <step>" is printed.  The tokens go through generate.extend, the function that continues sequences from the model's
caches and state.
"""

import argparse
import json
import os
import sys
from pathlib import Path

import torch

from . import _lib, generate


class TraceReplay:
    """One request at a time in row 0 of the model's state; the next one may start when the last has ended."""

    def __init__(self, model, device, max_tokens: int):
        self.model, self.device = model, device
        self.live, self.position = None, 0
        model.setup_caches(max_batch_size=1, max_seq_length=max_tokens)

    def step(self, entries, end):
        """-> float32 [wanted, vocab] on the host, or None when nothing is wanted."""
        rows = []
        for e in entries:
            if self.live is None:
                self.live, self.position = e["id"], 0
            if e["id"] != self.live:
                raise ValueError(f"request {e['id']} begins while {self.live} has not ended")
            n = len(e["tokens"])
            if n == 0:
                continue
            if self.position + n > self.model.max_seq_length:
                raise ValueError(f"request {e['id']} holds more tokens than the cache was sized for")
            tokens = torch.tensor([e["tokens"]], dtype=torch.int64, device=self.device)
            logits = generate.extend(self.model, tokens, self.position)
            self.position += n
            if e["want"]:
                rows.append(logits[0, torch.tensor(e["want"], device=self.device)].float())
        for name in end:
            if name == self.live:
                self.live = None
        return torch.cat(rows).cpu() if rows else None


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay a trace of token ids (JSON lines on standard input) and write logits.")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", required=True, choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    args = ap.parse_args(argv)

    _lib.load_seq(build_if_missing=True)
    if not torch.cuda.is_available():
        print("trace_run: no GPU", file=sys.stderr)
        return 2
    torch.backends.cuda.matmul.allow_tf32 = False  # float32 products in true float32
    device = "cuda:0"
    precision = torch.bfloat16 if args.dtype == "bfloat16" else torch.float32
    replay = TraceReplay(generate.load_model(args.model, device, precision), device, args.max_tokens)
    out = Path(args.out)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = replay.step(step["entries"], step.get("end", []))
        if logits is not None:
            part = out / f".{step['step']}.part"
            part.write_bytes(logits.numpy().astype("<f4").tobytes())
            os.replace(part, out / f"{step['step']}.f32")
        torch.cuda.synchronize()
        print(f"done {step['step']}", flush=True)
    return 0
