"""Inputs and comparisons shared by the op tests."""
import torch

from agentcontrolplane_amd.engine.batch import FlatBatch, SeqMeta

BF16, F32 = torch.bfloat16, torch.float32


def close(got, want, dtype, scale=1.0):
    tol = (2e-2 if dtype == BF16 else 3e-5) * scale
    err = (got.double().cpu() - want.double().cpu()).abs().max().item()
    assert err <= tol * max(1.0, want.abs().max().item()), err


def rand(*shape, dtype, device, seed=0, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dtype).to(device)


def make_batch(chunks, block, device, seed=0, spare=3):
    """chunks: [(ctx, new)].  Chunks of one token after cached ones are decode
    rows, as in the engine.  Pages are handed out in random order."""
    chunks = [c for c in chunks if c[1] > 1 or c[0] == 0] + [
        c for c in chunks if c[1] == 1 and c[0] > 0
    ]
    need = [-(-(ctx + new) // block) for ctx, new in chunks]
    order = torch.randperm(
        sum(need) + spare, generator=torch.Generator().manual_seed(seed)
    ).tolist()
    prefills, tables, lens = [], [], []
    for i, ((ctx, new), k) in enumerate(zip(chunks, need)):
        pages, order = order[:k], order[k:]
        if new == 1 and ctx > 0:
            tables.append(pages)
            lens.append(ctx + 1)
        else:
            prefills.append(SeqMeta(i, new, ctx + new, ctx, pages, True))
    width = max(map(len, tables), default=0)
    t = lambda x: torch.tensor(x, device=device)  # noqa: E731
    batch = FlatBatch(
        token_ids=torch.zeros(sum(n for _, n in chunks), dtype=torch.long, device=device),
        positions=t([ctx + k for ctx, new in chunks for k in range(new)]),
        slot_mapping=t([0]), prefills=prefills,
        num_prefill_tokens=sum(m.query_len for m in prefills),
        decode_seq_ids=list(range(len(tables))),
        decode_block_tables=t([p + [0] * (width - len(p)) for p in tables]) if tables else None,
        decode_seq_lens=t(lens) if lens else None,
        logit_rows=t([0]), sample_seq_ids=[],
    )
    return batch, chunks, [m.block_table for m in prefills] + tables, sum(need) + spare
