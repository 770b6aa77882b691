"""Replays traces: given token ids go through the engine's step, portion by portion, and chosen logits come out.

Steps are read from standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

Every entry brings a request's next tokens and the places among them whose logits are wanted; all entries of a step run
as one batch. Requests named in "end" give back what they hold. A step in which something is wanted writes
OUT/<step>.f32: little-endian floats [wanted, vocab] in the order of the entries and of their places. "done <step>" is
printed after every step. Nothing is sampled.
"""

from __future__ import annotations

import argparse
import json
import sys
from pathlib import Path

SLOTS = 4      # requests that may be live at once


def parse_args(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True, help="a checkpoint folder (config.json and model.safetensors)")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"],
                    help="bfloat16: as the engine serves the model; float32: everything in 32-bit")
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="most tokens that live requests hold at any time, each rounded up to whole pages: the size of the cache")
    return ap.parse_args(argv)


class Replay:
    def __init__(self, engine) -> None:
        self.engine = engine
        self.free = list(range(SLOTS))
        self.live: dict = {}          # id -> [slot, tokens held]

    def step(self, entries, end):
        """The logits wanted by the entries, in order (None when nothing is wanted)."""
        rows, want = [], []
        for e in entries:
            if not e["tokens"]:
                raise ValueError("an entry brings no tokens")
            if e["id"] not in self.live:
                if not self.free:
                    raise ValueError("more than %d requests are live" % SLOTS)
                self.live[e["id"]] = [self.free.pop(0), 0]
            slot, held = self.live[e["id"]]
            want += [(len(rows), k) for k in e["want"]]
            rows.append((slot, e["tokens"], held))
            self.live[e["id"]][1] = held + len(e["tokens"])
        logits = self.engine.step_logits(rows, want) if rows else None
        for name in end:
            slot, _ = self.live.pop(name)
            self.engine.seq_rm(slot)
            self.free.append(slot)
        return logits if want else None


def main(argv=None) -> int:
    args = parse_args(argv)
    from . import build, engine as E

    if not E.LIB_PATH.exists():
        build.build(library_only=True)
    n = max(args.max_tokens, 64)
    config = E.EngineConfig(n_ctx=n, n_seq_max=SLOTS, n_batch=n, n_ubatch=n,
                            kv_dtype=E.KV_F16 if args.dtype == "bfloat16" else E.KV_F32)
    out = Path(args.out)
    with E.Engine(args.model, config) as eng:
        replay = Replay(eng)
        for line in sys.stdin:
            if not line.strip():
                continue
            step = json.loads(line)
            logits = replay.step(step["entries"], step.get("end", []))
            if logits is not None:
                (out / ("%d.f32" % step["step"])).write_bytes(logits.astype("<f4").tobytes())
            print("done %d" % step["step"], flush=True)
    return 0
