"""Grouped attention without rotation: capped scores, a window that keeps the first
tokens, a sink in the softmax, and keys and values that another layer may own.

    q, k, v = W h + b;  query head n uses key/value head n // (heads / kv_heads)
    s_ij = softcap * tanh(scale * q_i . k_j / softcap)
    i sees j:  j <= i and (i - j < window or j < keep_first)
    out_i = sum_j exp(s_ij) v_j / (exp(sink) + sum_j exp(s_ij))

Query/key and value heads are zero-padded to the kernels' sizes at load time;
padding stays zero through every product.  The whole sequence stays in the pages:
a layer that borrows keys may have the longer window.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import torch

from .. import ops
from ..engine.batch import FlatBatch
from ..engine.config import GroupedAttentionSpec
from .layout import Get, pad_to


class GroupedAttention:
    def __init__(self, spec: GroupedAttentionSpec, width: int, tp_rank: int, tp_world: int):
        if spec.heads % spec.kv_heads:
            raise ValueError("kv_heads must divide heads")
        if spec.kv_heads % tp_world:
            raise ValueError("TP degree must divide the key/value head count")
        self.spec, self.width = spec, width
        self.heads, self.kv_heads = spec.heads // tp_world, spec.kv_heads // tp_world
        self.tp_rank = tp_rank
        self.d, self.v = ops.latent_head(spec.dim), ops.latent_head(spec.vdim)
        self.w_in: torch.Tensor = None   # [q | k | v rows, width]; q alone on borrowed keys
        self.bias: Optional[torch.Tensor] = None
        self.sink: Optional[torch.Tensor] = None   # fp32
        self.w_out: torch.Tensor = None

    # ------------------------------------------------------------- weights

    def _parts(self) -> List[Tuple[str, int, int, int]]:
        """(tensor, heads of the whole model, head size, padded head size)"""
        s = self.spec
        parts = [("q", s.heads, s.dim, self.d)]
        if s.kv_from is None:
            parts += [("k", s.kv_heads, s.dim, self.d), ("v", s.kv_heads, s.vdim, self.v)]
        return parts

    def shapes(self) -> List[Tuple[str, Tuple[int, ...]]]:
        """Checkpoint tensors of the whole (unsharded) mixer."""
        s, out = self.spec, []
        for name, heads, size, _ in self._parts():
            out.append((name, (heads * size, self.width)))
            if s.bias:
                out.append((name + ".b", (heads * size,)))
        if s.sink:
            out.append(("sink", (s.heads,)))
        return out + [("o", (self.width, s.heads * s.vdim))]

    def _mine(self, t: torch.Tensor, heads: int) -> torch.Tensor:
        """This rank's of ``heads`` along dim 0."""
        n = heads * self.kv_heads // self.spec.kv_heads
        return t[self.tp_rank * n : (self.tp_rank + 1) * n]

    def load(self, get: Get, p: str) -> None:
        s, rows, biases = self.spec, [], []
        for name, heads, size, padded in self._parts():
            w = self._mine(get(p + name).view(heads, size, self.width), heads)
            rows.append(pad_to(w, len(w), padded, self.width).flatten(0, 1))
            if s.bias:
                b = self._mine(get(p + name + ".b").view(heads, size), heads)
                biases.append(pad_to(b, len(b), padded).flatten())
        self.w_in = torch.cat(rows).contiguous()
        if s.bias:
            self.bias = torch.cat(biases)
        if s.sink:
            self.sink = self._mine(get(p + "sink"), s.heads).float().contiguous()
        o = get(p + "o").view(self.width, s.heads, s.vdim).transpose(0, 1)
        o = self._mine(o, s.heads).transpose(0, 1)
        self.w_out = pad_to(o, self.width, self.heads, self.v).flatten(1).contiguous()

    def export(self, p: str) -> Dict[str, torch.Tensor]:
        """Inverse of load() (unsharded models)."""
        s, out, at = self.spec, {}, 0
        for name, heads, size, padded in self._parts():
            n = heads * padded
            w = self.w_in[at : at + n].view(heads, padded, self.width)[:, :size]
            out[p + name] = w.reshape(heads * size, self.width)
            if s.bias:
                out[p + name + ".b"] = self.bias[at : at + n].view(heads, padded)[:, :size].flatten()
            at += n
        if s.sink:
            out[p + "sink"] = self.sink.to(self.w_in.dtype)
        o = self.w_out.view(self.width, s.heads, self.v)[:, :, : s.vdim]
        out[p + "o"] = o.reshape(self.width, s.heads * s.vdim)
        return out

    # --------------------------------------------------------------- cache

    def new_cache(self, num_blocks: int, block_size: int, dtype, device):
        """Keys and values, or None for a layer that uses another one's.
        Uninitialised: a row is written before any query can see it."""
        if self.spec.kv_from is not None:
            return None
        shape = (num_blocks, block_size, self.kv_heads)
        return tuple(torch.empty(*shape, n, dtype=dtype, device=device) for n in (self.d, self.v))

    @property
    def cache_row(self) -> int:
        """Cached elements per token."""
        return 0 if self.spec.kv_from is not None else self.kv_heads * (self.d + self.v)

    # ------------------------------------------------------------- forward

    def forward(self, h: torch.Tensor, batch: FlatBatch,
                cache: Tuple[torch.Tensor, torch.Tensor]) -> torch.Tensor:
        """h [N, width] -> this rank's part of [N, width]."""
        s, N = self.spec, h.shape[0]
        proj = ops.linear(h, self.w_in, self.bias)
        row, at = proj.stride(0), self.heads * self.d
        q = proj.as_strided((N, self.heads, self.d), (row, self.d, 1))
        if s.kv_from is None:
            k = proj.as_strided((N, self.kv_heads, self.d), (row, self.d, 1), at)
            at += self.kv_heads * self.d
            v = proj.as_strided((N, self.kv_heads, self.v), (row, self.v, 1), at)
            ops.cache_keys_values(k, v, batch.slot_mapping, *cache)
        out = torch.empty(N, self.heads, self.v, dtype=h.dtype, device=h.device)
        ops.grouped_attention(
            q, *cache, batch, s.scale, s.softcap, s.window, s.keep_first, self.sink, out
        )
        return ops.linear(out.view(N, -1), self.w_out)
