"""Grouped attention over paged keys and values, with the parts a design picks.

    q, k, v = conv(W h + b);  query head n uses key/value head n // (heads / kv_heads)
    q, k = rmsnorm(.) w, per head or over all heads, rotated;  v = rmsnorm(v)
    q_i *= 1 + coef ln(floor((i + 1) / every) + 1),  times a learned factor per head
    s_ij = scale * q_i . k_j,  mixed over the heads:  s_h <- sum_g T[h, g] s_g
    s_ij = cap(s_ij) + bias[bucket(i - j)]
    i sees j:  j <= i and (i - j < window or j < keep_first)
               and floor(i / chunk) = floor(j / chunk)
    out_i = sum_j exp(s_ij) v_j / (exp(sink) + sum_j exp(s_ij))
         or sum_j sigmoid(s_ij + offset) v_j,  times sigmoid(W_g h) per head

Every line but the first product is optional (GroupedAttentionSpec); the keys and
values may be another layer's.  What a design does to q, k and v between the
projection and the cache is one op (attention_inputs); the short convolutions' last
inputs are a ring by position in the sequence's state slot.

Query/key and value heads are zero-padded to the kernels' sizes at load time;
padding stays zero through every product.  The whole sequence stays in the pages:
a layer that borrows keys may have the longer window.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

from .. import ops
from ..engine.batch import FlatBatch
from ..engine.config import DistanceBias, GroupedAttentionSpec
from .layout import Get, pad_to, pair_halves, round_up, unpair_halves


def distance_buckets(spec: DistanceBias) -> torch.Tensor:
    """Bucket of every distance up to the first one in the last bucket, to which all
    larger ones belong."""
    half = spec.buckets // 2
    out = list(range(half))
    while not out or out[-1] < spec.buckets - 1:
        grow = math.log(len(out) / half) / math.log(spec.reach / half) if half else math.inf
        # distances that begin a bucket exactly must not fall below it by rounding
        step = math.floor(grow * (spec.buckets - half) + 1e-9) if half else spec.buckets
        out.append(min(spec.buckets - 1, half + step))
    return torch.tensor(out)


class GroupedAttention:
    def __init__(self, spec: GroupedAttentionSpec, width: int, eps: float,
                 tp_rank: int, tp_world: int):
        if spec.heads % spec.kv_heads:
            raise ValueError("kv_heads must divide heads")
        if spec.kv_heads % tp_world:
            raise ValueError("TP degree must divide the key/value head count")
        if spec.kv_from is not None and (spec.conv or spec.qk_norm or spec.rotary):
            raise ValueError("borrowed keys are used as their owner cached them")
        if tp_world > 1 and (spec.row_norm or spec.talk):
            raise ValueError("norms and score mixes over all heads need them on one rank")
        if spec.row_norm and (spec.qk_norm or spec.conv):
            raise ValueError("a norm over all heads goes with neither head norms nor convolutions")
        if spec.chunk and spec.keep_first:
            raise ValueError("chunks keep no first tokens")
        self.spec, self.width, self.eps = spec, width, eps
        self.heads, self.kv_heads = spec.heads // tp_world, spec.kv_heads // tp_world
        self.tp_rank = tp_rank
        self.d, self.v = ops.latent_head(spec.dim), ops.latent_head(spec.vdim)
        self.out_dim = self.heads * self.v
        #: channels of q | k | v (q alone on borrowed keys)
        kv = 0 if spec.kv_from is not None else self.kv_heads * (self.d + self.v)
        self.channels = self.heads * self.d + kv
        #: is there more between the projection and the cache than a copy?
        self.shaped = bool(spec.conv or spec.qk_norm or spec.row_norm or spec.v_norm
                           or spec.rotary or spec.q_temp or spec.head_temp)
        self.w_in: torch.Tensor = None   # [q | k | v | head gates | beside rows, width]
        self.beside_at: Optional[Tuple[int, int]] = None  # first row and rows of beside
        self.bias: Optional[torch.Tensor] = None
        self.conv: Optional[torch.Tensor] = None       # [taps, channels]
        self.q_norm = self.k_norm = None               # [d], or of all heads
        self.w_out: torch.Tensor = None
        self.out_bias: Optional[torch.Tensor] = None   # on the first rank
        # fp32
        self.sink = self.temp = None                   # [heads]
        self.talk: Optional[torch.Tensor] = None       # [heads, heads]
        self.rel = self.offset = None                  # [buckets, heads], [heads]
        self.dist_bias: Optional[torch.Tensor] = None  # [heads, distances], offset included
        self.cos_sin: Optional[torch.Tensor] = None    # set by the model if spec.rotary

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
            if s.conv:
                out.append((name + ".conv", (heads * size, s.conv)))
        if s.qk_norm:
            out += [("q.norm", (s.dim,)), ("k.norm", (s.dim,))]
        if s.row_norm:
            out += [("q.norm", (s.heads * s.dim,)), ("k.norm", (s.kv_heads * s.dim,))]
        if s.talk:
            out.append(("talk", (s.heads, s.heads)))
        if s.distance_bias:
            out.append(("rel", (s.distance_bias.buckets, s.heads)))
        if s.sigmoid:
            out.append(("pb", (s.heads,)))
        if s.head_temp:
            out.append(("temp", (s.heads,)))
        if s.sink:
            out.append(("sink", (s.heads,)))
        if s.head_gate:
            out.append(("g", (s.heads, self.width)))
        out.append(("o", (self.width, s.heads * s.vdim)))
        return out + ([("o.b", (self.width,))] if s.out_bias else [])

    def _mine(self, t: torch.Tensor, heads: int) -> torch.Tensor:
        """This rank's of ``heads`` along dim 0."""
        n = heads * self.kv_heads // self.spec.kv_heads
        return t[self.tp_rank * n : (self.tp_rank + 1) * n]

    def _laid_out(self, t: torch.Tensor, name: str, heads: int, size: int,
                  padded: int) -> torch.Tensor:
        """[heads * size, k] -> this rank's heads, rotated dims paired, padded."""
        t = self._mine(t.view(heads, size, -1), heads)
        if self.spec.rotary and name != "v":
            t = pair_halves(t, self.spec.rotary.dims, 1)
        return pad_to(t, t.shape[0], padded, t.shape[2]).flatten(0, 1)

    def _restored(self, t: torch.Tensor, name: str, size: int, padded: int) -> torch.Tensor:
        """Inverse of _laid_out() (unsharded)."""
        t = t.reshape(-1, padded, t.shape[-1])[:, :size]
        if self.spec.rotary and name != "v":
            t = unpair_halves(t, self.spec.rotary.dims, 1)
        return t.reshape(-1, t.shape[-1])

    def _head_norm(self, t: torch.Tensor) -> torch.Tensor:
        if self.spec.rotary:
            t = pair_halves(t, self.spec.rotary.dims)
        return pad_to(t, self.d).contiguous()

    def load(self, get: Get, p: str,
             beside: Optional[Tuple[torch.Tensor, torch.Tensor]] = None) -> None:
        """``beside``: rows and bias of another product of the same input."""
        s, rows, biases, taps, row_norms = self.spec, [], [], [], {}
        for part in self._parts():
            if s.row_norm and part[0] != "v":
                w = get(p + part[0] + ".norm").unsqueeze(1)
                row_norms[part[0]] = self._laid_out(w, *part).flatten().contiguous()
            rows.append(self._laid_out(get(p + part[0]), *part))
            if s.bias:
                biases.append(self._laid_out(get(p + part[0] + ".b").unsqueeze(1), *part))
            if s.conv:
                taps.append(self._laid_out(get(p + part[0] + ".conv"), *part))
        if s.head_gate:
            gate = self._mine(get(p + "g"), s.heads)
            rows.append(pad_to(gate, round_up(self.heads, 16), self.width))
        if beside:
            self.beside_at = (sum(len(r) for r in rows), beside[0].shape[0])
            rows.append(pad_to(beside[0], round_up(beside[0].shape[0], 16), self.width))
        self.w_in = torch.cat(rows).contiguous()
        if s.bias or beside:
            self.bias = self.w_in.new_zeros(self.w_in.shape[0])
        if s.bias:
            self.bias[: self.channels] = torch.cat(biases).flatten()
        if beside:
            at, n = self.beside_at
            self.bias[at : at + n] = beside[1]
        if s.conv:
            self.conv = torch.cat(taps).t().contiguous()
        if s.qk_norm:
            self.q_norm = self._head_norm(get(p + "q.norm"))
            self.k_norm = self._head_norm(get(p + "k.norm"))
        if s.row_norm:
            self.q_norm, self.k_norm = row_norms["q"], row_norms["k"]
        if s.talk:
            self.talk = get(p + "talk").float().contiguous()

        def per_head(name):
            return self._mine(get(p + name), s.heads).float().contiguous()

        if s.sink:
            self.sink = per_head("sink")
        if s.head_temp:
            self.temp = per_head("temp")
        if s.sigmoid:
            self.offset = per_head("pb")
        if s.distance_bias:
            self.rel = self._mine(get(p + "rel").t(), s.heads).t().float()
            buckets = distance_buckets(s.distance_bias).to(self.rel.device)
            self.dist_bias = self.rel[buckets].t().contiguous()
        elif s.sigmoid:
            self.dist_bias = torch.zeros(self.heads, 1, device=self.offset.device)
        if s.sigmoid:
            self.dist_bias = self.dist_bias + self.offset.unsqueeze(1)
        o = get(p + "o").view(self.width, s.heads, s.vdim).transpose(0, 1)
        o = self._mine(o, s.heads).transpose(0, 1)
        self.w_out = pad_to(o, self.width, self.heads, self.v).flatten(1).contiguous()
        if s.out_bias and self.tp_rank == 0:
            self.out_bias = get(p + "o.b").contiguous()

    def export(self, p: str) -> Dict[str, torch.Tensor]:
        """Inverse of load() (unsharded models)."""
        s, dt, out, at = self.spec, self.w_in.dtype, {}, 0
        for name, heads, size, padded in self._parts():
            n = heads * padded
            out[p + name] = self._restored(self.w_in[at : at + n], name, size, padded)
            if s.bias:
                b = self.bias[at : at + n].unsqueeze(1)
                out[p + name + ".b"] = self._restored(b, name, size, padded).flatten()
            if s.row_norm and name != "v":
                t = (self.q_norm if name == "q" else self.k_norm).unsqueeze(1)
                out[p + name + ".norm"] = self._restored(t, name, size, padded).flatten()
            if s.conv:
                taps = self.conv[:, at : at + n].t()
                out[p + name + ".conv"] = self._restored(taps, name, size, padded)
            at += n
        if s.qk_norm:
            for name, t in (("q.norm", self.q_norm), ("k.norm", self.k_norm)):
                t = t[: s.dim]
                out[p + name] = unpair_halves(t, s.rotary.dims) if s.rotary else t
        if s.distance_bias:
            out[p + "rel"] = self.rel.to(dt)
        for name, t in (("sink", self.sink), ("temp", self.temp), ("pb", self.offset),
                        ("talk", self.talk)):
            if t is not None:
                out[p + name] = t.to(dt)
        if s.head_gate:
            out[p + "g"] = self.w_in[at : at + s.heads]
        o = self.w_out.view(self.width, s.heads, self.v)[:, :, : s.vdim]
        out[p + "o"] = o.reshape(self.width, s.heads * s.vdim)
        if s.out_bias:
            out[p + "o.b"] = self.out_bias
        return out

    def beside(self) -> Tuple[torch.Tensor, torch.Tensor]:
        at, n = self.beside_at
        return self.w_in[at : at + n], self.bias[at : at + n]

    # ----------------------------------------------------- pages and state

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

    def new_state(self, num_slots: int, dtype, device) -> Optional[torch.Tensor]:
        """The convolutions' last inputs per slot; uninitialised: nothing before a
        sequence's start is read."""
        if not self.spec.conv:
            return None
        return torch.empty(num_slots, self.spec.conv, self.channels, dtype=dtype, device=device)

    def state_bytes(self, itemsize: int) -> int:
        return self.spec.conv * self.channels * itemsize

    # ------------------------------------------------------------- forward

    def attend(self, h: torch.Tensor, batch: FlatBatch, cache: Tuple[torch.Tensor, torch.Tensor],
               ring: Optional[torch.Tensor], out: torch.Tensor) -> Optional[torch.Tensor]:
        """h [N, width] -> out [N, heads * v] (row-strided): the heads ahead of W_o.
        Returns the product beside the mixer's, if there is one."""
        s, N = self.spec, h.shape[0]
        proj = ops.linear(h, self.w_in, self.bias)
        row, at = proj.stride(0), self.heads * self.d
        q = proj.as_strided((N, self.heads, self.d), (row, self.d, 1))
        if self.shaped:
            q = ops.attention_inputs(
                proj[:, : self.channels], self.heads, s.dim, s.vdim, *cache, batch, self.eps,
                conv=self.conv, ring=ring, q_norm=self.q_norm, k_norm=self.k_norm,
                v_norm=s.v_norm, cos_sin=self.cos_sin, head_mult=self.temp,
                q_temp=(s.q_temp.coef, s.q_temp.every) if s.q_temp else None,
            )
        elif s.kv_from is None:
            k = proj.as_strided((N, self.kv_heads, self.d), (row, self.d, 1), at)
            at += self.kv_heads * self.d
            v = proj.as_strided((N, self.kv_heads, self.v), (row, self.v, 1), at)
            ops.cache_keys_values(k, v, batch.slot_mapping, *cache)
        gate = proj[:, self.channels : self.channels + self.heads] if s.head_gate else None
        out = out.as_strided((N, self.heads, self.v), (out.stride(0), self.v, 1))
        ops.grouped_attention(
            q, *cache, batch, s.scale, s.softcap, s.window, s.keep_first, self.sink, out,
            bias=self.dist_bias, sigmoid=s.sigmoid, gate=gate, chunk=s.chunk, talk=self.talk,
        )
        if self.beside_at is None:
            return None
        at, n = self.beside_at
        return proj[:, at : at + n]

    def mix(self, h: torch.Tensor, batch: FlatBatch, cache: Tuple[torch.Tensor, torch.Tensor]):
        """h [N, width] -> the heads ahead of W_o [N, heads * v] and, if there is one, the
        product beside the mixer's."""
        out = torch.empty(h.shape[0], self.out_dim, dtype=h.dtype, device=h.device)
        return out, self.attend(h, batch, cache, None, out)

    def forward(self, h: torch.Tensor, batch: FlatBatch,
                cache: Tuple[torch.Tensor, torch.Tensor]) -> torch.Tensor:
        """h [N, width] -> this rank's part of [N, width]."""
        return ops.linear(self.mix(h, batch, cache)[0], self.w_out, self.out_bias)
