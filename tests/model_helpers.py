"""Running a checkpoint through the engine in chosen portions, for the model tests."""
import torch

from agentcontrolplane_amd.engine.config import EngineConfig
from agentcontrolplane_amd.engine.engine import InferenceEngine


def make_engine(path, device, dtype="float32", start=False, **kw):
    kw = {"num_kv_blocks": 96, "max_model_len": 1024, "max_batch_size": 8, **kw}
    return InferenceEngine(
        EngineConfig(model="auto", checkpoint_path=path, dtype=dtype, device=device, **kw),
        start=start,
    )


def tokens(n, cfg, seed=0):
    g = torch.Generator().manual_seed(100 + seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def feed(replay, rid, ids, cuts, end=True):
    """Run one request alone in the given portions; logits of every token."""
    rows, at = [], 0
    for c in cuts:
        part = ids[at : at + c]
        at += c
        rows.append(replay.step(
            [{"id": rid, "tokens": part, "want": list(range(len(part)))}],
            [rid] if end and at == len(ids) else [],
        ))
    return torch.cat(rows)


def assert_close(got, want, dtype="float32"):
    """Logits, mean taken off: rms error per position beside their spread.  A
    fault is of order 1 where it strikes; bf16 rounding reaches some tenths at
    single positions of these small random models."""
    d = got.double() - want.double()
    d = d - d.mean(-1, keepdim=True)
    err = d.pow(2).mean(-1).sqrt() / want.double().std()
    most, typical = (1e-4, 1e-5) if dtype == "float32" else (0.5, 0.03)
    assert err.max() < most, (err.max().item(), err.argmax().item())
    if len(err) > 40:
        assert err.median() < typical, err.median().item()


CUTS = {
    "whole": lambda n: [n],
    "tokens": lambda n: [1] * n,
    "twos": lambda n: [2] * (n // 2) + [1] * (n % 2),
    "pages": lambda n: [16] * (n // 16) + ([n % 16] if n % 16 else []),
    "changing": lambda n: _fit([3, 17, 1, 31, 2, 1, 1, 15, 64, 5], n),
    "prompt_then_tokens": lambda n: [n - 40] + [1] * 40,
}


def _fit(pattern, n):
    out, i = [], 0
    while sum(out) < n:
        out.append(min(pattern[i % len(pattern)], n - sum(out)))
        i += 1
    return out
