"""Prefill and decode throughput of a model design beside the dense GQA model
(Llama) of equal size: same width, head count, feed-forward, vocabulary and
number of layer runs, random weights.

Both run through the engine's scheduler, block manager and forward (decode steps
replay captured graphs).  The two sides of a workload are timed in turn, several
rounds, and each side's best round counts.
"""
from __future__ import annotations

import dataclasses
import time
from typing import Dict, List, Tuple

import torch

from ..engine.config import PRESETS, EngineConfig, ModelConfig
from ..engine.engine import InferenceEngine
from ..engine.request import InferenceRequest, SamplingParams

#: (sequences, tokens each) of one prefill step
PREFILL = [(1, 1024), (1, 4096), (1, 8192), (16, 512)]
#: (sequences, cached tokens each) of one decode step
DECODE = [(1, 4096), (16, 1024), (64, 1024), (64, 4096), (256, 1024)]


def dense_twin(cfg: ModelConfig) -> ModelConfig:
    """The Llama model of cfg's size."""
    return ModelConfig(
        name=cfg.name + "-dense", vocab_size=cfg.vocab_size, hidden_size=cfg.hidden_size,
        intermediate_size=cfg.intermediate_size, num_layers=len(cfg.layer_runs),
        num_heads=cfg.num_heads, num_kv_heads=min(8, cfg.num_heads), head_dim=128,
        max_position=cfg.max_position, rms_eps=cfg.rms_eps, dtype=cfg.dtype,
    )


class Side:
    """One model in its engine, with sequences laid out by the scheduler."""

    def __init__(self, cfg: ModelConfig, device: str, max_len: int, pool_tokens: int,
                 max_batch: int):
        PRESETS.setdefault(cfg.name, cfg)
        self.engine = InferenceEngine(
            EngineConfig(
                model=cfg.name, device=device, max_model_len=max_len,
                num_kv_blocks=-(-pool_tokens // EngineConfig.kv_block_size),
                max_batch_size=max_batch,
            ),
            start=False,
        )
        self.engine.scheduler.continuation_cache = False
        m = self.engine.model
        # decode workloads attend over tokens that were never prefilled
        for c in getattr(m, "caches", None) or m.k_caches + m.v_caches:
            c.normal_(0.0, 0.5)
        for c in getattr(m, "states", ()):
            c.normal_(0.0, 0.1)

    def _sequence(self, tokens: int):
        ids = [(7 * i) % 250 for i in range(tokens)]
        return self.engine.scheduler.add_request(
            InferenceRequest(ids, SamplingParams(max_tokens=1))
        )

    def step(self, n: int, tokens: int, decode: bool):
        """A zero-argument step to time, and its clean-up."""
        sched = self.engine.scheduler
        seqs = [self._sequence(tokens) for _ in range(n)]
        if decode:
            for s in seqs:  # cached so far: reserve the pages, keep their contents
                sched.waiting.remove(s)
                sched.running.append(s)
                sched.reserve(s)
                self.engine.bm.append_tokens(s.seq_id, tokens - 1)
                s.num_processed = tokens - 1
            portions = [(s, 1, [0]) for s in seqs]
        else:
            portions = [(s, tokens, [tokens - 1]) for s in seqs]
        batch, _ = sched.schedule_portions(portions)

        def done():
            for s in seqs:
                sched.finish_seq(s, "stop")

        return (lambda: self.engine.forward_batch(batch)), done


def _time(fn, iters: int, cuda: bool) -> float:
    if cuda:
        torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(iters):
        fn()
    if cuda:
        torch.cuda.synchronize()
    return (time.perf_counter() - t0) / iters


def run(name: str, device: str, prefill: List[Tuple[int, int]] = PREFILL,
        decode: List[Tuple[int, int]] = DECODE, iters: int = 5, rounds: int = 3) -> Dict:
    cfg = PRESETS[name]
    cuda = device.startswith("cuda")
    work = [(n, t, False) for n, t in prefill] + [(n, t, True) for n, t in decode]
    max_len = max(t for _, t, _ in work) + 16
    pool = max(n * (t + 16) for n, t, _ in work)
    most = max(n for n, _, _ in work)
    sides = {
        "design": Side(dataclasses.replace(cfg), device, max_len, pool, most),
        "dense": Side(dense_twin(cfg), device, max_len, pool, most),
    }
    rows = []
    for n, tokens, is_decode in work:
        best = {k: float("inf") for k in sides}
        steps = {k: s.step(n, tokens, is_decode) for k, s in sides.items()}
        for fn, _ in steps.values():
            _time(fn, 2, cuda)
        for _ in range(rounds):
            for k, (fn, _) in steps.items():
                best[k] = min(best[k], _time(fn, iters, cuda))
        for _, done in steps.values():
            done()
        made = n if is_decode else n * tokens
        rows.append({
            "step": "decode" if is_decode else "prefill", "sequences": n, "tokens": tokens,
            **{f"{k}_ms": round(1e3 * b, 3) for k, b in best.items()},
            **{f"{k}_tok_s": round(made / b) for k, b in best.items()},
        })
    return {
        "design": name,
        "dense": dense_twin(cfg).name,
        "layer_runs": len(cfg.layer_runs),
        "cache_bytes_per_token": {
            k: s.engine.model.kv_block_bytes(1) for k, s in sides.items()
        },
        "state_bytes_per_sequence": {
            k: getattr(s.engine.model, "state_slot_bytes", 0) for k, s in sides.items()
        },
        "workloads": rows,
    }
