"""Replay token steps through the engine and write the logits.

Reads one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3],
                             "want": [0, 2]}], "end": []}

Every entry brings the next tokens of one request; all entries of a line
are one batch of LLMEngine.step, against what earlier steps left in the
cache. `want` lists the places among an entry's tokens whose logits are
written, as little-endian f32 [wanted, vocab], to OUT/<step>.f32. `end`
lists requests that are finished after the step. After each step a line
"done <step>" is printed. Nothing is sampled.
"""

from __future__ import annotations

import argparse
import json
import sys
from pathlib import Path

import torch

from ..models import load_pretrained
from .engine import LLMEngine, _Seq

MAX_LIVE = 4  # requests that are live at the same time


class TraceReplay:
    def __init__(self, engine: LLMEngine, out: Path):
        self.engine = engine
        self.out = out
        self.live: dict[str, _Seq] = {}

    def run(self, line: dict) -> None:
        work, want = [], []
        for e in line["entries"]:
            rid = e["id"]
            if rid not in self.live:
                self.live[rid] = _Seq(seq_id=len(self.live), prompt_ids=[])
            if e["tokens"]:
                work.append((self.live[rid], e["tokens"]))
                want.append(e.get("want", []))
        if work:
            logits = self.engine.step(work, want)
            if logits is not None:
                data = logits.float().cpu().numpy().astype("<f4")
                (self.out / f"{line['step']}.f32").write_bytes(
                    data.tobytes())
        for rid in line.get("end", []):
            self.engine.release(self.live.pop(rid))


def main(argv: list[str] | None = None) -> int:
    ap = argparse.ArgumentParser(
        prog="trace_run",
        description="Replay token steps through a model, writing logits.")
    ap.add_argument("--model", required=True,
                    help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", default="bfloat16",
                    choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, type=Path)
    ap.add_argument("--max-tokens", required=True, type=int,
                    help="most tokens that live requests hold together")
    args = ap.parse_args(argv)

    if not torch.cuda.is_available():
        print("trace_run needs a GPU", file=sys.stderr)
        return 1
    # products in float32 stay float32
    torch.backends.cuda.matmul.allow_tf32 = False
    model = load_pretrained(args.model, device="cuda:0",
                            dtype=getattr(torch, args.dtype))
    blk = LLMEngine.BLK
    engine = LLMEngine(model, max_batch_size=MAX_LIVE,
                       max_model_len=args.max_tokens,
                       num_blocks=(args.max_tokens + blk - 1) // blk)
    args.out.mkdir(parents=True, exist_ok=True)
    replay = TraceReplay(engine, args.out)
    for text in sys.stdin:
        if not text.strip():
            continue
        line = json.loads(text)
        replay.run(line)
        print(f"done {line['step']}", flush=True)
    return 0
