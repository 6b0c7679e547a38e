"""Op dispatch.

Two implementations of every engine op:

- ``reference`` — plain PyTorch fp32, runs on CPU.  The numerics oracle for
  every HIP kernel test and the compute path for CPU-only engine tests.
- ``hip`` — hand-written CDNA4 HIP kernels (csrc/*.hip) through the in-tree
  ``_C`` extension.  The ONLY path on a GPU: if a tensor is on cuda and the
  extension is missing, ops raise instead of silently falling back, so a GPU
  run that passes is guaranteed to have run the native kernels.
"""
from __future__ import annotations

from typing import NamedTuple, Optional

import torch

_HIP = None
_HIP_ERR: Exception | None = None


def _hip():
    global _HIP, _HIP_ERR
    if _HIP is None and _HIP_ERR is None:
        try:
            from . import hip as m

            _HIP = m
        except Exception as e:  # pragma: no cover
            _HIP_ERR = e
    if _HIP is None:
        raise RuntimeError(
            f"HIP ops extension not available on a GPU tensor path: {_HIP_ERR}\n"
            "Build it with: python build_ext.py (PYTORCH_ROCM_ARCH=gfx950)"
        )
    return _HIP


def _impl(t: torch.Tensor):
    if t.is_cuda:
        return _hip()
    from . import reference as m

    return m


import os

# Measured A/B (tools/gemm_bench.py, profiles/r01_gemm_ab.md): the TunableOp-
# tuned hipBLASLt stream-K kernels hold 1.3-1.6 PF on every engine projection
# shape; the hand-written 8-phase kernel (csrc/gemm_bf16.hip) reaches 1.1 PF
# (zero LDS conflicts, barrier/issue-stall bound).  The library stays the
# default; set ACP_GEMM_MIN_M to route M >= threshold to the custom kernel.
_GEMM_MIN_M = int(os.environ.get("ACP_GEMM_MIN_M", str(1 << 30)))


def linear(x, w, bias=None):
    """x[*, K] @ w[N, K]^T (+ bias[N]) → [*, N].  Large-M bf16 shapes go to the
    hand-written 8-phase MFMA GEMM (csrc/gemm_bf16.hip); everything else
    (decode-sized M, ragged shards, CPU) to torch.nn.functional.linear."""
    if (
        x.is_cuda
        and bias is None
        and x.dtype == torch.bfloat16
        and x.dim() == 2
        and x.shape[0] >= _GEMM_MIN_M
        and w.shape[0] % 256 == 0
        and w.shape[1] % 128 == 0
    ):
        return _hip().gemm_bf16(x, w)
    return torch.nn.functional.linear(x, w, bias)


def linear_add_(y, x, w):
    """y += x @ w^T in one GEMM."""
    return y.addmm_(x, w.t())


def rmsnorm(x, weight, eps: float = 1e-5):
    return _impl(x).rmsnorm(x, weight, eps)


def fused_add_rmsnorm(x, residual, weight, eps: float = 1e-5):
    """returns (normed, new_residual) where new_residual = x + residual."""
    return _impl(x).fused_add_rmsnorm(x, residual, weight, eps)


def rope_and_cache(q, k, v, positions, slot_mapping, k_cache, v_cache, cos_sin):
    """Apply rotary embedding to q,k in place and scatter k,v into the paged
    cache at slot_mapping.  q:[N, Hq, D] k/v:[N, Hkv, D]."""
    return _impl(q).rope_and_cache(q, k, v, positions, slot_mapping, k_cache, v_cache, cos_sin)


def attention_prefill(q, k_cache, v_cache, block_table, seq_len, ctx_len, scale):
    """Causal attention for ONE sequence's prefill chunk (test/oracle entry).
    q: [Lq, Hq, D]; KV read from the paged cache; ctx_len = tokens already
    cached before this chunk (the chunk's causal offset)."""
    return _impl(q).attention_prefill(q, k_cache, v_cache, block_table, seq_len, ctx_len, scale)


def attention_prefill_batch(q, k_cache, v_cache, batch, scale, out=None):
    """Causal attention for ALL prefill chunks of a FlatBatch in one launch.
    q: [num_prefill_tokens, Hq, D]."""
    return _impl(q).attention_prefill_batch(q, k_cache, v_cache, batch, scale, out)


def attention_decode_batch(q, k_cache, v_cache, batch, scale, out=None):
    """One-token-per-sequence paged attention.  q: [B, Hq, D]."""
    return _impl(q).attention_decode_batch(q, k_cache, v_cache, batch, scale, out)


def swiglu(gate_up):
    """gate_up: [N, 2*I] (gate | up interleaved as two halves) → [N, I]."""
    return _impl(gate_up).swiglu(gate_up)


# ------------------------------------------------ fp32-residual norms, GLU, gates


def layernorm(x, weight, eps: float, dtype):
    """Layer norm without bias of an fp32 residual [N, K] -> dtype."""
    return _impl(x).layernorm(x, weight, eps, dtype)


class Depth(NamedTuple):
    """States of a depth average: X_0 (the embedding output) and every layer's result."""

    states: torch.Tensor   # [layers + 1, N, K] fp32
    coef: torch.Tensor     # [layers, layers + 1] fp32: row i weighs the states after layer i
    partial: torch.Tensor  # [DEPTH_AHEAD, N, K] fp32 workspace

    @staticmethod
    def new(coef: torch.Tensor, N: int, K: int) -> "Depth":
        planes = torch.empty(
            coef.shape[1] + DEPTH_AHEAD, N, K, dtype=torch.float32, device=coef.device
        )
        return Depth(planes[: coef.shape[1]], coef, planes[coef.shape[1] :])


#: sums the first layer of a block prepares for the block's others (csrc/residual_norm.h)
DEPTH_AHEAD = 3


def residual_norm(x, y, eps: float, y_norm=None, x_norm=None, out=None, *, center=True,
                  offset: float = 0.0, mult: float = 1.0, depth: Optional[Depth] = None,
                  layer: int = 0, x_norm2=None, out2=None, experts=None, gate=None):
    """x += mult * y, or x += mult * rmsnorm(y) * y_norm, in the fp32 residual x, where
    ``experts`` (rows [N, k, K], weights [N, k] fp32) joins y as
    sum_j weights[:, j] * rows[:, j] and then ``gate`` [N, K] (row-strided) multiplies it
    by its sigmoid; then, with ``depth``, x is filed as layer ``layer``'s state and replaced by
    sum_j coef[layer, j] * states[j] (layers in order: later ones use sums made by
    earlier ones); then out = norm(x) * x_norm, or x itself without x_norm.  The norm
    of x is a layer norm, an RMS norm if not ``center``; ``offset`` is added to the
    norm weights.  out2 is the same norm under the weight x_norm2."""
    return _impl(x).residual_norm(
        x, y, eps, y_norm, x_norm, out, center, offset, mult, depth, layer, x_norm2, out2,
        experts, gate,
    )


def embed_positions(token_ids, positions, table, cos_sin, x, copy=None, scale: float = 1.0):
    """x = copy = scale * table[token] plus, with cos_sin [2, P, ceil(K / 2)], sin (even
    entries) and cos (odd entries) of the position's angles; x, copy fp32 [N, K]."""
    return _impl(x).embed_positions(token_ids, positions, table, cos_sin, x, copy, scale)


def softcap(logits, cap):
    """cap * tanh(logits / cap) in fp32; the logits in fp32 without a cap."""
    return logits.float() if cap is None else _impl(logits).softcap(logits, cap)


def clamped_glu(gate_up, limit: float, alpha: float, offset: float, out, cubic: float = 0.0):
    """gate_up [N, 2I] (row-strided halves) -> out [N, I] (row-strided):
    g * sigmoid(alpha (g + cubic g^3)) * (u + offset), g capped at limit, u at +-limit."""
    return _impl(gate_up).clamped_glu(gate_up, limit, alpha, offset, out, cubic)


def side_gate(x, y, gate, token_ids, table, offset: int):
    """The fp32 residual x + y (x itself may be reused for it) and
    gelu_tanh(gate (x + y)) * table[token, offset : offset + D]: [N, D]."""
    return _impl(x).side_gate(x, y, gate, token_ids, table, offset)


# ------------------------------------------------------------ latent attention

#: latent sizes the MFMA kernels are built for; larger ones run the plain kernel
LATENT_RANKS = (64, 128, 256, 384, 512)


def latent_rank(kv_rank: int) -> int:
    """The padded latent size kernels and caches use for kv_rank."""
    for r in LATENT_RANKS:
        if kv_rank <= r:
            return r
    return -(-kv_rank // 64) * 64


#: query/key and value head sizes of the expanded prefill kernel
LATENT_HEADS = (64, 128, 256)


def latent_head(dim: int) -> int:
    """The padded per-head size for dim."""
    for n in LATENT_HEADS:
        if dim <= n:
            return n
    return -(-dim // 64) * 64


def latent_inputs(kv, norm_w, eps: float, kv_rank: int, rot_dim: int, rank: int,
                  positions, slot_mapping, cos_sin, cache, q=None, q_norm=None, q_rank=0):
    """kv [N, kv_rank + rot_dim] (row-strided): RMS-norm the latent, rotate the
    key part (interleaved pairs), scatter [latent -> rank | rotated] rows into
    cache [blocks, block, row].  With q [N, K] (low-rank query, row-strided; its
    columns past q_rank are zero padding) returns rmsnorm(q) * q_norm."""
    return _impl(kv).latent_inputs(
        kv, norm_w, eps, kv_rank, rot_dim, rank, positions, slot_mapping, cos_sin, cache,
        q, q_norm, q_rank,
    )


def head_linear(x, w, out, gate=None):
    """out[n, h] = w[h] @ x[n, h], times sigmoid(gate[n, h]) if given.
    x [N, H, K], w [H, O, K], out [N, H, O]; x, out, gate row-strided."""
    return _impl(x).head_linear(x, w, out, gate)


def latent_attention(q, q_rot, cos_sin, rot_dim: int, cache, batch, scale: float, window,
                     row0: int = 0, skip=(), sink=None):
    """Softmax attention of absorbed queries over cached rows (``sink`` [H], fp32, or None
    joins the denominator), for a FlatBatch's token rows row0.. except the prefill chunks in ``skip`` (left undefined).
    q [N, H, rank] and its part q_rot [N, H, rot] still to be rotated by the
    row's position; values are a cache row's first ``rank`` dims.
    window = visible keys per query, None = all.  Returns [N, H, rank]."""
    return _impl(q).latent_attention(
        q, q_rot, cos_sin, rot_dim, cache, batch, scale, window, row0, skip, sink
    )


def can_expand(t, d: int, v: int, rot: int) -> bool:
    """Is there a kernel for expanded keys and values of these padded sizes?"""
    return t.is_cuda and _hip().can_expand(t.dtype, d, v, rot)


def latent_expanded_prefill(q, w_ukv, gate, cos_sin, rot_dim: int, cache, batch, chunks,
                            rank: int, scale: float, window, out, sink=None):
    """The prefill chunks ``chunks`` with keys and values expanded from their
    cached latents by w_ukv [H*d + H*v, rank]; q [N, H, d + rot] not rotated.
    Writes the chunks' rows of out [N, H, v], gated."""
    _hip().latent_expanded_prefill(
        q, w_ukv, gate, cos_sin, rot_dim, cache, batch, chunks, rank, scale, window, out, sink
    )


# ---------------------------------------- grouped attention: caps, windows, sinks


def cache_keys_values(k, v, slot_mapping, k_cache, v_cache):
    """Scatter k [N, G, d], v [N, G, e] (row-strided) into paged caches
    [blocks, block, G, d or e]."""
    return _impl(k).cache_keys_values(k, v, slot_mapping, k_cache, v_cache)


def attention_inputs(proj, heads: int, dim: int, vdim: int, k_cache, v_cache, batch, eps: float,
                     *, conv=None, ring=None, q_norm=None, k_norm=None, v_norm: bool = False,
                     cos_sin=None, head_mult=None, q_temp=None):
    """From projected rows [N, q | k | v channels] (row-strided; heads padded from dim and
    vdim to the caches' d and e) to queries [N, heads, d], which are returned, and keys
    and values in their cache slots (batch.slot_mapping).  In this order, each optional:

    conv [taps, channels]: causal convolution per channel; the last inputs of a
        sequence are kept by position in its slot of ``ring`` [slots, taps, channels]
    q_norm, k_norm [d], v_norm: RMS norm per head over dim or vdim; [heads * d] and
        [G * d]: over all heads at once (no conv, no v_norm)
    cos_sin [2, P, n]: rotate a query's and key's first n pairs (2i, 2i + 1)
    head_mult [heads] fp32, q_temp (coef, every): queries times the head's factor, and
        times 1 + coef ln(floor((p + 1) / every) + 1) at position p"""
    return _impl(proj).attention_inputs(
        proj, heads, dim, vdim, k_cache, v_cache, batch, eps, conv, ring, q_norm, k_norm,
        v_norm, cos_sin, head_mult, q_temp,
    )


def grouped_attention(q, k_cache, v_cache, batch, scale: float, cap, window, keep_first: int,
                      sink, out, bias=None, sigmoid: bool = False, gate=None, chunk=None,
                      talk=None):
    """Attention of a FlatBatch's rows over the paged cache; query head n uses
    key/value head n // (H / G).  ``talk`` [H, H] (fp32, of values that the
    model's dtype holds) mixes the scores over the heads: head h's are
    sum_g talk[h, g] * head g's.  Scores are capped if ``cap``; a query sees
    itself and the ``window`` - 1 tokens before it (None = all) and the ``keep_first``
    first tokens, with ``chunk`` (no keep_first) only those of its own chunk, position
    // chunk; ``sink`` [H] (fp32) or None joins the softmax denominator.
    ``bias`` [H, D] (fp32) adds bias[h, min(distance, D - 1)] to the capped scores;
    ``sigmoid``: weights are the scores' sigmoids, not a softmax; ``gate`` [N, H]
    (row-strided) multiplies a head's output by its sigmoid.
    q [N, H, d], out [N, H, e], both row-strided."""
    return _impl(q).grouped_attention(
        q, k_cache, v_cache, batch, scale, cap, window, keep_first, sink, out, bias, sigmoid,
        gate, chunk, talk,
    )


# -------------------------------------------------------------------- experts


def moe_route(h, router, bias, top: int, sigmoid: bool = False, scale: float = 1.0):
    """The ``top`` experts with the largest logits router @ h + bias (fp32) of every row:
    ids [N, top] int32 and scale * the softmax over the chosen logits [N, top] fp32.
    ``sigmoid``: the choice is by sigmoid(router @ h) + bias, the weights are
    scale * the chosen sigmoids over their sum."""
    return _impl(h).moe_route(h, router, bias, top, sigmoid, scale)


def moe_experts(h, gate_up, down, ids, glu):
    """Every chosen expert's GLU of its row: h [N, K], gate_up [E, 2I, K], down [E, W, I],
    ids [N, k] -> [N, k, W].  ``glu`` has limit, alpha, offset and cubic."""
    return _impl(h).moe_experts(h, gate_up, down, ids, glu)


# ----------------------------------------------------------------- delta rule


def gated_delta(qkv, conv, b, z, A_log, dt_bias, gate, norm, eps: float, unit_eps: float,
                kv_heads: int, state, conv_state, batch, gate_silu: bool = False):
    """Gated delta rule over a FlatBatch's rows, each sequence from the state in its
    slot (zero at position 0), which is advanced.  Row-strided inputs: qkv
    [N, 2*G*D + H*V] before the convolution, b [N, H] before its sigmoid, z [N, H*D]
    or [N, H] (one decay per head) the decays' input, gate [N, H*V] before its sigmoid or
    silu.  conv [channels, taps]; fp32: A_log [H], dt_bias like z, norm [V], state
    [slots, H, D, V]; conv_state [slots, taps, channels], the last convolution inputs in a
    ring by position.  Returns [N, H*V]: normed per head and gated."""
    return _impl(qkv).gated_delta(
        qkv, conv, b, z, A_log, dt_bias, gate, norm, eps, unit_eps, kv_heads, state,
        conv_state, batch, gate_silu,
    )


def softmax_sample(logits, temperatures, top_ks, top_ps, gen, mask=None,
                   uniforms=None, mask_map=None):
    """Batch sampling: temperature/top-k/top-p with optional boolean vocab
    masks (constrained decoding; compact [M, V] rows + mask_map [B]
    indirection for BPE-scale vocabularies) and optional precomputed
    per-row uniforms (per-request seeded generators).  Returns [B] long."""
    return _impl(logits).softmax_sample(
        logits, temperatures, top_ks, top_ps, gen, mask, uniforms, mask_map
    )
