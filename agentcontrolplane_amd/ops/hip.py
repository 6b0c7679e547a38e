"""GPU op dispatch into the hand-written CDNA4 kernels (csrc/*.hip).

No fallbacks: a cuda-tensor call that cannot reach a kernel raises, so a
passing GPU run proves the native path ran (the round-end loader check
looks for agentcontrolplane_amd/_C.so in the process maps).
"""
from __future__ import annotations

import torch

from .. import _C  # in-tree extension; ImportError surfaces via ops.__init__


def rmsnorm(x, weight, eps: float = 1e-5):
    out = torch.empty_like(x)
    _C.rmsnorm(out, x, weight, eps)
    return out


def fused_add_rmsnorm(x, residual, weight, eps: float = 1e-5):
    out = torch.empty_like(x)
    _C.fused_add_rmsnorm(out, residual, x, weight, eps)  # residual updated in place
    return out, residual


def rope_and_cache(q, k, v, positions, slot_mapping, k_cache, v_cache, cos_sin):
    _C.rope_cache(q, k, v, positions, slot_mapping, k_cache, v_cache, cos_sin)
    return q, k


def attention_prefill(q, k_cache, v_cache, block_table, seq_len, ctx_len, scale):
    """Single-sequence entry (tests): wrap into a one-seq batched call."""
    from ..engine.batch import FlatBatch, SeqMeta

    meta = SeqMeta(
        seq_id=0, query_len=q.shape[0], seq_len=seq_len, ctx_len=ctx_len,
        block_table=list(block_table), needs_logits=True,
    )
    dummy = torch.empty(0)
    batch = FlatBatch(
        token_ids=torch.empty(q.shape[0], device=q.device),
        positions=dummy, slot_mapping=dummy, prefills=[meta],
        num_prefill_tokens=q.shape[0], decode_seq_ids=[],
        decode_block_tables=None, decode_seq_lens=None,
        logit_rows=dummy, sample_seq_ids=[],
    )
    return attention_prefill_batch(q, k_cache, v_cache, batch, scale)


import os

_PREFILL_IMPL = os.environ.get("ACP_PREFILL_IMPL", "mfma")  # mfma | v0


def _attn_out(q):
    return torch.empty(q.shape, dtype=q.dtype, device=q.device)


def attention_prefill_batch(q, k_cache, v_cache, batch, scale, out=None):
    if out is None:
        out = _attn_out(q)
    if _PREFILL_IMPL == "mfma":
        meta = batch.prefill_meta(tile_q=128)
        _C.prefill_attn_mfma(
            out, q, k_cache, v_cache, meta.block_tables, meta.seq_lens, meta.ctx_lens,
            meta.row_starts, meta.tile_seq, meta.tile_q0, scale,
        )
    else:
        meta = batch.prefill_meta(tile_q=64)
        _C.prefill_attn(
            out, q, k_cache, v_cache, meta.block_tables, meta.seq_lens, meta.ctx_lens,
            meta.row_starts, meta.tile_seq, meta.tile_q0, scale,
        )
    return out


def attention_decode_batch(q, k_cache, v_cache, batch, scale, out=None):
    if out is None:
        out = _attn_out(q)
    _C.decode_attn(
        out, q, k_cache, v_cache, batch.decode_tables_i32(), batch.decode_lens_i32(),
        scale,
    )
    return out


def attention_decode_raw(q, k_cache, v_cache, block_tables, seq_lens, scale):
    out = _attn_out(q)
    _C.decode_attn(
        out, q, k_cache, v_cache, block_tables.int().contiguous(),
        seq_lens.int().contiguous(), scale,
    )
    return out


def gemm_bf16(x, w):
    out = torch.empty((x.shape[0], w.shape[0]), dtype=x.dtype, device=x.device)
    _C.gemm_bf16(out, x.contiguous(), w)
    return out


def swiglu(gate_up):
    inter = gate_up.shape[-1] // 2
    out = torch.empty(
        (*gate_up.shape[:-1], inter), dtype=gate_up.dtype, device=gate_up.device
    )
    _C.swiglu(out, gate_up)
    return out


# ------------------------------------------------ fp32-residual norms, GLU, gates


def layernorm(x, weight, eps: float, dtype):
    out = torch.empty(x.shape, dtype=dtype, device=x.device)
    _C.residual_norm(
        x, None, None, weight, out, eps, True, 0.0, 1.0, None, None, None, 0, None, None, None,
        None, None,
    )
    return out


def residual_norm(x, y, eps: float, y_norm=None, x_norm=None, out=None, center=True,
                  offset=0.0, mult=1.0, depth=None, layer=0, x_norm2=None, out2=None,
                  experts=None, gate=None):
    states, coef, partial = depth or (None, None, None)
    rows, weights = experts or (None, None)
    _C.residual_norm(
        x, y, y_norm, x_norm, out, eps, center, offset, mult, states, coef, partial, layer,
        x_norm2, out2, rows, weights, gate,
    )


def embed_positions(token_ids, positions, table, cos_sin, x, copy=None, scale=1.0):
    _C.embed_positions(x, copy, token_ids, positions, table, cos_sin, scale)


def softcap(logits, cap):
    out = torch.empty(logits.shape, dtype=torch.float32, device=logits.device)
    _C.softcap(out, logits, cap)
    return out


def clamped_glu(gate_up, limit: float, alpha: float, offset: float, out, cubic=0.0):
    _C.clamped_glu(out, gate_up, limit, alpha, offset, cubic)


#: up to this many tokens the fused side_gate kernel beats the GEMM route
_SIDE_GATE_TOKENS = 256


def side_gate(x, y, gate, token_ids, table, offset: int):
    from . import linear

    if x.shape[0] <= _SIDE_GATE_TOKENS and x.shape[1] % 8 == 0:
        s = torch.empty(x.shape[0], gate.shape[0], dtype=gate.dtype, device=x.device)
        x_new = torch.empty_like(x)
        _C.side_gate(s, x_new, x, y, gate, token_ids, table, offset)
        return x_new, s
    xt = None if gate.dtype == torch.float32 else torch.empty_like(y)
    _C.add_to_residual(x, y, xt)
    s = linear(x if xt is None else xt, gate)
    _C.gelu_gate(s, token_ids, table, offset)
    return x, s


# ------------------------------------------------------------ latent attention

_NO_WINDOW = 1 << 30
_MAX_SPLIT = 32


def latent_inputs(kv, norm_w, eps: float, kv_rank: int, rot_dim: int, rank: int,
                  positions, slot_mapping, cos_sin, cache, q=None, q_norm=None, q_rank=0):
    cq = None if q is None else torch.empty(q.shape, dtype=q.dtype, device=q.device)
    _C.latent_inputs(
        cache, kv, norm_w, positions, slot_mapping, cos_sin, eps, kv_rank, rot_dim, rank,
        cq, q, q_norm, q_rank,
    )
    return cq


def head_linear(x, w, out, gate=None):
    _C.head_linear(out, x, w, gate)
    return out


def _latent_attn(out, q, q_rot, cos_sin, rot_dim, cache, tables, seq_lens, prefill, tiles,
                 mg, max_keys, scale, window, mfma, sink):
    """One launch over prefill tiles (prefill = their metadata) or decode
    rows.  Few tiles split their keys over several workgroups."""
    n_split = 1
    if mfma:
        keys = min(max_keys, window)
        # workgroups that fill the chip: the tiles of a wide latent take a CU's LDS
        fill = 256 if q.shape[2] >= 256 else 512
        n_split = max(1, min(_MAX_SPLIT, fill // tiles, -(-keys // 128)))
    part = ml = None
    if n_split > 1:
        rows = q.shape[0] * q.shape[1]
        part = torch.empty(n_split * rows * q.shape[2], dtype=torch.float32, device=q.device)
        # rows no tile covers (skipped chunks) must merge to nothing
        new = torch.empty if prefill is None else torch.zeros
        ml = new(2 * n_split * rows, dtype=torch.float32, device=q.device)
    m = prefill
    _C.latent_attn(
        out, q, q_rot, cos_sin, rot_dim, cache, tables, seq_lens,
        *((m.ctx_lens, m.row_starts, m.tile_seq, m.tile_q0) if m else (None,) * 4),
        part, ml, sink, scale, window, mg, n_split, mfma,
    )


def latent_attention(q, q_rot, cos_sin, rot_dim: int, cache, batch, scale: float, window,
                     row0: int = 0, skip=(), sink=None):
    from . import LATENT_RANKS

    N, H, rank = q.shape
    out = torch.empty(N, H, rank, dtype=q.dtype, device=q.device)
    window = window or _NO_WINDOW
    mfma = q.dtype == torch.bfloat16 and rank in LATENT_RANKS and q_rot.shape[2] == 64
    most = 4 if rank <= 256 else 2
    P = batch.num_prefill_tokens - row0
    common = (cos_sin, rot_dim, cache)
    chunks = tuple(i for i in range(len(batch.prefills)) if i not in skip)
    if chunks:
        meta = batch.prefill_meta(
            16 * most if mfma else 1, rows_per_token=H, only=chunks, row_base=row0
        )
        _latent_attn(
            out[:P], q[:P], q_rot[:P], *common, meta.block_tables, meta.seq_lens, meta,
            meta.tile_seq.numel(), most, max(batch.prefills[i].seq_len for i in chunks),
            scale, window, mfma, sink,
        )
    if batch.num_decode:
        mg = 1 if H <= 16 else 2 if H <= 32 else most
        tables = batch.decode_tables_i32()
        _latent_attn(
            out[P:], q[P:], q_rot[P:], *common, tables, batch.decode_lens_i32(), None,
            batch.num_decode * -(-H // (16 * mg)), mg,
            tables.shape[1] * cache.shape[1], scale, window, mfma, sink,
        )
    return out


#: expanded keys and values built at a time
_EXPAND_BYTES = 2 << 30


def can_expand(dtype, d: int, v: int, rot: int) -> bool:
    from . import LATENT_HEADS

    return dtype == torch.bfloat16 and rot == 64 and d in LATENT_HEADS and v in LATENT_HEADS


def _expansion_groups(batch, chunks, window: int, bytes_per_key: int):
    groups, at = [], 0
    for i in chunks:
        m = batch.prefills[i]
        keys = (m.seq_len - max(0, m.ctx_len - window + 1)) * bytes_per_key
        if not groups or at + keys > _EXPAND_BYTES:
            groups.append([])
            at = 0
        groups[-1].append(i)
        at += keys
    return [tuple(g) for g in groups]


def latent_expanded_prefill(q, w_ukv, gate, cos_sin, rot_dim: int, cache, batch, chunks,
                            rank: int, scale: float, window, out, sink=None):
    from . import linear

    window = window or _NO_WINDOW
    row = cache.shape[2]
    groups = batch.memo(
        ("expansion_groups", chunks, window, w_ukv.shape[0]),
        lambda: _expansion_groups(batch, chunks, window, 2 * w_ukv.shape[0]),
    )
    for group in groups:
        meta = batch.prefill_meta(128, only=group, window=window)
        rows = torch.empty(meta.num_keys, row, dtype=q.dtype, device=q.device)
        _C.latent_gather(
            rows, cache, meta.block_tables, meta.seq_lens, meta.key_first, meta.key_starts,
            meta.max_keys,
        )
        _C.latent_prefill(
            out, q, linear(rows[:, :rank], w_ukv), rows[:, rank:], gate, cos_sin, rot_dim,
            meta.seq_lens, meta.ctx_lens, meta.row_starts, meta.tile_seq, meta.tile_q0,
            meta.key_first, meta.key_starts, sink, scale, window,
        )


# ---------------------------------------- grouped attention: caps, windows, sinks

_PLAIN, _DECODE, _PREFILL, _TALK_DECODE, _TALK_PREFILL = range(5)


def cache_keys_values(k, v, slot_mapping, k_cache, v_cache):
    _C.cache_keys_values(k_cache, v_cache, k, v, slot_mapping)


def _conv_rows(batch):
    """Per row of a step: rows of its sequence right before it, and its state slot.
    None, slots: every row is alone in its sequence's step."""
    if not batch.prefills:
        return None, batch.decode_state_slots
    P, meta = batch.num_prefill_tokens, batch.prefill_meta(16)
    ctx, slots = torch.stack([meta.ctx_lens, meta.state_slots]).repeat_interleave(
        meta.seq_lens - meta.ctx_lens, 1, output_size=P
    )
    back = batch.positions[:P].int() - ctx
    if batch.num_decode:
        back = torch.cat([back, back.new_zeros(batch.num_decode)])
        slots = torch.cat([slots, batch.decode_state_slots])
    return back, slots.contiguous()


def _ring_rows(batch, taps: int):
    """The last rows of every portion, as many as a ring holds."""
    rows, at = [], 0
    for m in batch.prefills:
        at += m.query_len
        rows.extend(range(at - min(m.query_len, taps), at))
    rows.extend(range(at, at + batch.num_decode))
    if batch._stager is not None:
        return batch._stager.tensor(f"ring_rows{taps}", rows, "int32")
    return torch.tensor(rows, dtype=torch.int32, device=batch.positions.device)


def attention_inputs(proj, heads, dim, vdim, k_cache, v_cache, batch, eps, conv, ring, q_norm,
                     k_norm, v_norm, cos_sin, head_mult, q_temp):
    q = torch.empty(proj.shape[0], heads, k_cache.shape[3], dtype=proj.dtype, device=proj.device)
    back = states = ring_rows = None
    if conv is not None:
        back, states = batch.memo("conv_rows", lambda: _conv_rows(batch))
        if batch.prefills:
            taps = conv.shape[0]
            ring_rows = batch.memo(("ring_rows", taps), lambda: _ring_rows(batch, taps))
    coef, every = q_temp or (0.0, 0.0)
    _C.attention_inputs(
        q, k_cache, v_cache, proj, batch.positions, batch.slot_mapping, dim, vdim, eps, conv,
        ring, back, states, ring_rows, ring_rows is None, q_norm, k_norm, v_norm, cos_sin,
        head_mult, coef, every,
    )
    return q


def grouped_attention(q, k_cache, v_cache, batch, scale: float, cap, window, keep_first: int,
                      sink, out, bias=None, sigmoid=False, gate=None, chunk=None, talk=None):
    from . import LATENT_HEADS

    H, d, v, G = q.shape[1], q.shape[2], out.shape[2], k_cache.shape[2]
    rest = (scale, cap or 0.0, window or _NO_WINDOW, chunk or _NO_WINDOW, keep_first, sigmoid)
    bf16 = q.dtype == torch.bfloat16
    if talk is None:
        tiled = bf16 and d in LATENT_HEADS and v in LATENT_HEADS and not (sigmoid and cap)
        kinds, tile = ((_DECODE, _PREFILL) if tiled else (_PLAIN, _PLAIN)), 128
    else:
        tiled = bf16 and not (sigmoid or cap or keep_first) and all(
            t is None for t in (sink, bias, gate))
        tile = _C.talk_prefill_tokens(H, G, d, v, k_cache.shape[1]) if tiled else 0
        tiled = tiled and _C.talk_decode_fits(H, G, d, v)
        kinds = (_TALK_DECODE if tiled else _PLAIN, _TALK_PREFILL if tile else _PLAIN)
    P = batch.num_prefill_tokens

    def gates(r):
        return None if gate is None else gate[r]

    if batch.prefills:
        if kinds[1] == _TALK_PREFILL:
            meta = batch.prefill_meta(tile, chunk=chunk or _NO_WINDOW)
        else:
            meta = batch.prefill_meta(1 if kinds[1] == _PLAIN else tile)
        _C.grouped_attn(
            out[:P], q[:P], k_cache, v_cache, meta.block_tables, meta.seq_lens, meta.ctx_lens,
            meta.row_starts, meta.tile_seq, meta.tile_q0, sink, bias, gates(slice(0, P)), talk,
            None, None, *rest, kinds[1], 1, 1,
        )
    if not batch.num_decode:
        return
    tables, rows = batch.decode_tables_i32(), batch.num_decode * H
    gm, n_split, part, ml = 1, 1, None, None
    # keys a row may see
    keys = min(tables.shape[1] * k_cache.shape[1], rest[2] + keep_first, rest[3])
    if kinds[0] == _TALK_DECODE:  # a workgroup has all heads, and 4 waves with 32 keys each
        n_split = max(1, min(_MAX_SPLIT, 1024 // batch.num_decode, -(-keys // 128)))
    elif kinds[0] == _DECODE:
        most = 8 if d + v <= 256 else 4  # query heads a workgroup holds
        gm = next((n for n in (1, 2, 4) if n >= min(H // G, most)), most)
        # workgroups that fill the chip; every split has work for its 16 lane groups
        groups = batch.num_decode * G * -(-(H // G) // gm)
        n_split = max(1, min(_MAX_SPLIT, 1024 // groups, -(-keys // 128)))
    if n_split > 1:
        part = torch.empty(n_split * rows * v, dtype=torch.float32, device=q.device)
        ml = torch.empty(2 * n_split * rows, dtype=torch.float32, device=q.device)
    _C.grouped_attn(
        out[P:], q[P:], k_cache, v_cache, tables, batch.decode_lens_i32(), None, None, None,
        None, sink, bias, gates(slice(P, None)), talk, part, ml, *rest,
        kinds[0], gm, n_split,
    )


# -------------------------------------------------------------------- experts


def moe_route(h, router, bias, top: int, sigmoid=False, scale=1.0):
    ids = torch.empty(h.shape[0], top, dtype=torch.int32, device=h.device)
    weights = torch.empty(h.shape[0], top, dtype=torch.float32, device=h.device)
    _C.moe_route(ids, weights, h, router, bias, sigmoid, scale)
    return ids, weights


#: average rows per expert from which the tiled product is faster (its weights are read
#: once, however many rows there are)
_TILED_ROWS = 12


def moe_experts(h, gate_up, down, ids, glu):
    (N, k), E, inner = ids.shape, gate_up.shape[0], down.shape[2]
    n, device = N * k, h.device
    act = torch.empty(n, inner, dtype=h.dtype, device=device)
    rows = torch.empty(N, k, down.shape[1], dtype=h.dtype, device=device)
    form = (glu.limit, glu.alpha, glu.offset, glu.cubic)
    perm = offsets = tile_expert = tile_row = None
    kind, tt = 0, 1
    if h.dtype == torch.bfloat16:
        tiled = n >= _TILED_ROWS * E and gate_up.shape[2] % 128 == 0 and inner % 128 == 0
        kind, tt = (2, 1) if tiled else (1, 1 if n <= 8 * E else 2)
        perm = torch.empty(n, dtype=torch.int32, device=device)
        offsets = torch.empty(E + 2, dtype=torch.int32, device=device)
        if tiled:
            tiles = torch.empty(2, n // _C.EXPERT_TILE + E, dtype=torch.int32, device=device)
            tile_expert, tile_row = tiles
        _C.moe_group(perm, offsets, tile_expert, tile_row, ids, E)
    grouped = (ids, perm, offsets, tile_expert, tile_row)
    _C.experts_linear(act, h, gate_up, *grouped, True, *form, kind, tt)
    _C.experts_linear(rows.view(n, -1), act, down, *grouped, False, *form, kind, tt)
    return rows


# ----------------------------------------------------------------- delta rule


def _step_threads(D: int, V: int, workgroups: int) -> int:
    """Threads of a decode workgroup: at most 16 rows of the state per thread, fewer
    while the workgroups do not fill the chip."""
    columns = V // 4 if V % 4 == 0 else V
    rows = 16 if workgroups >= 512 else 4
    for n in (256, 512):
        if n >= columns and n // columns * rows >= D:
            return n
    return 1024


def gated_delta(qkv, conv, b, z, A_log, dt_bias, gate, norm, eps, unit_eps, kv_heads,
                state, conv_state, batch, gate_silu=False):
    H, D, V = state.shape[1:]
    out = torch.empty(gate.shape, dtype=qkv.dtype, device=qkv.device)
    P = batch.num_prefill_tokens

    def rows(r):
        return (out[r], qkv[r], conv, b[r], z[r], A_log, dt_bias, gate[r], norm, state,
                conv_state)

    if batch.prefills:
        meta = batch.prefill_meta(16)
        seqs = len(batch.prefills)

        def space(n, dtype=torch.float32):
            return torch.empty(P * n, dtype=dtype, device=qkv.device)

        # two columns a lane once one still fills the chip's SIMDs
        cpl = 2 if seqs * H * V >= 4 * 4096 else 1
        _C.delta_prompts(
            *rows(slice(0, P)), meta.seq_lens, meta.state_slots, kv_heads, eps, unit_eps,
            gate_silu, meta.ctx_lens, meta.row_starts, meta.tile_seq, meta.tile_q0,
            space(qkv.shape[1], qkv.dtype), space(3 * kv_heads),
            None if z.shape[1] == H else space(H * D), space(H * V), cpl,
        )
    if batch.num_decode:
        _C.delta_step(
            *rows(slice(P, None)), batch.decode_lens_i32(), batch.decode_state_slots, kv_heads,
            eps, unit_eps, gate_silu, _step_threads(D, V, batch.num_decode * H),
        )
    return out


def softmax_sample(logits, temperatures, top_ks, top_ps, gen, mask=None,
                   uniforms=None, mask_map=None):
    B, V = logits.shape
    out = torch.empty(B, dtype=torch.long, device=logits.device)
    if uniforms is None:
        uniforms = torch.rand(B, device=logits.device, generator=gen)
    if V > 512:
        # BPE-scale vocab: LDS radix-select kernel, bf16 logits unconverted
        # (csrc/sampling_fullvocab.hip); masks are compact [M, V] rows with
        # mask_map [B] indirection (-1 = unconstrained row)
        if logits.dtype not in (torch.bfloat16, torch.float32):
            logits = logits.float()
        if mask is not None and mask_map is None:
            mask_map = torch.arange(B, dtype=torch.int32, device=logits.device)
        _C.sample_fullvocab(
            out, logits.contiguous(), temperatures.float().contiguous(),
            top_ks.long().contiguous(), top_ps.float().contiguous(),
            uniforms.contiguous(),
            mask.contiguous() if mask is not None else None,
            mask_map.contiguous() if mask is not None else None,
        )
        return out
    _C.sample(
        out, logits.float().contiguous(), temperatures.float().contiguous(),
        top_ks.long().contiguous(), top_ps.float().contiguous(),
        uniforms.contiguous(), mask.contiguous() if mask is not None else None,
    )
    return out
