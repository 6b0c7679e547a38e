"""Trace replay: run given token ids through the engine step by step and write
the logits asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}], "end": []}

Each entry brings a request's next tokens; ``want`` are the places among them
whose logits are written to OUT/<step>.f32 ([wanted, vocab], little-endian
fp32, in entry order).  ``end`` names requests whose cache is given back.  After
every step a line ``done <step>`` is printed.  Nothing is sampled.

The steps run through the engine's own scheduler, block manager and forward (a
decode-only step replays the captured graph), only the choice of portions is the
trace's.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, List, Tuple

import torch

from .config import EngineConfig
from .engine import InferenceEngine
from .request import InferenceRequest, SamplingParams
from .scheduler import Sequence

#: the most requests a trace keeps live
MAX_LIVE = 4


class TraceReplay:
    def __init__(self, engine: InferenceEngine):
        self.engine = engine
        self.engine.scheduler.continuation_cache = False  # an ended request frees its pages
        self._live: Dict[str, Sequence] = {}

    def step(self, entries: List[dict], end: List[str]) -> torch.Tensor:
        """Run one step; returns the wanted logits [wanted, vocab] (CPU fp32)."""
        sched = self.engine.scheduler
        portions: List[Tuple[Sequence, int, List[int]]] = []
        for e in entries:
            seq = self._live.get(e["id"])
            if seq is None:
                seq = sched.add_request(InferenceRequest([], SamplingParams(max_tokens=1)))
                self._live[e["id"]] = seq
            seq.prompt_ids.extend(e["tokens"])
            if e["tokens"]:
                portions.append((seq, len(e["tokens"]), e["want"]))
        out = torch.empty(0, self.engine.mcfg.vocab_size)
        if portions:
            batch, places = sched.schedule_portions(portions)
            logits = self.engine.forward_batch(batch)
            row_of = {place: row for row, place in enumerate(places)}
            rows = [row_of[n, k] for n, (_, _, want) in enumerate(portions) for k in want]
            if rows:
                out = logits[torch.tensor(rows, device=logits.device)].float().cpu()
            elif logits.is_cuda:
                torch.cuda.synchronize()
        for rid in end:
            sched.finish_seq(self._live.pop(rid), "stop")
        return out


def build_engine(model: str, dtype: str, max_tokens: int, device: str) -> InferenceEngine:
    block = EngineConfig.kv_block_size
    return InferenceEngine(
        EngineConfig(
            model="auto", checkpoint_path=model, dtype=dtype, device=device,
            kv_block_size=block, num_kv_blocks=-(-max_tokens // block),
            max_model_len=max_tokens, max_batch_size=MAX_LIVE,
        ),
        start=False,
    )


def main(argv=None) -> int:
    p = argparse.ArgumentParser(prog="trace_run", description="replay a token trace")
    p.add_argument("--model", required=True, help="folder with config.json and safetensors")
    p.add_argument("--dtype", choices=["bfloat16", "float32"], required=True)
    p.add_argument("--out", required=True, help="folder for <step>.f32")
    p.add_argument("--max-tokens", type=int, required=True,
                   help="size of the cache pool in tokens")
    p.add_argument("--device", default="cuda")
    args = p.parse_args(argv)
    os.makedirs(args.out, exist_ok=True)
    replay = TraceReplay(build_engine(args.model, args.dtype, args.max_tokens, args.device))
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = replay.step(step["entries"], step.get("end", []))
        if logits.shape[0]:
            logits.numpy().astype("<f4").tofile(
                os.path.join(args.out, f"{step['step']}.f32")
            )
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
