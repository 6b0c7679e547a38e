"""Latent attention: one low-rank latent and one shared rotated key part are
cached per token; keys and values are linear in the latent.

    c      = rmsnorm(W_dkv h)[:kv_rank]           cached
    k_rot  = rotate(W_dkv h)[kv_rank:]            cached, shared by the heads
    score  = (q_nope . W_uk c + rotate(q_rot) . k_rot) * scale
    out    = sigmoid(W_g h) * sum_j p_j W_uv c_j

The query may be low-rank, the head gate absent, and a learned logit per head may
join the softmax denominator.  The rotation pairs dimension 2i with 2i + 1; a design
that pairs i with i + rot_dim/2 has its weight rows reordered at load time.

Two equal evaluations.  *Absorbed*: q' = W_uk^T q_nope, so a score is one dot
product with the cached row and the weighted sum is taken over latents, W_uv
applied once per query.  It reads one short row per key for all heads: decode
and short portions.  *Expanded*: keys and values are built per head once and
shared by many queries, which costs fewer products per (query, key) pair: long
prompt chunks.

Layout.  The kernels want 16-byte aligned rows and whole MFMA tiles, so weights
are laid out with zero rows at load time: a query head is
[dim -> d | rot_dim -> rot], a cache row [kv_rank -> rank | rot_dim -> rot], a
value head vdim -> v.  Padding stays exactly zero through every product.

The mixer works on sections of a fused input projection and writes a slice of a
fused output projection's input, both owned by the layer.
"""
from __future__ import annotations

from typing import Dict, List, Tuple

import torch

from .. import ops
from ..engine.batch import FlatBatch
from ..engine.config import LatentAttentionSpec
from .layout import Get, pad_to, pair_halves, round_up, unpair_halves


class LatentAttention:
    def __init__(self, spec: LatentAttentionSpec, width: int, eps: float,
                 tp_rank: int, tp_world: int):
        if spec.heads % tp_world:
            raise ValueError("TP degree must divide the head count")
        if spec.rot_dim % 2:
            raise ValueError("rot_dim must be even")
        self.spec, self.width, self.eps = spec, width, eps
        self.heads = spec.heads // tp_world
        self.head0 = tp_rank * self.heads
        self.d = ops.latent_head(spec.dim)
        self.rot = round_up(spec.rot_dim, 64)
        self.v = ops.latent_head(spec.vdim)
        self.rank = ops.latent_rank(spec.kv_rank)
        self.row = self.rank + self.rot          # cache row
        self.q_dim = self.heads * (self.d + self.rot)
        self.q_rank = round_up(spec.q_rank, 16) if spec.q_rank else 0
        self.out_dim = self.heads * self.v
        # set by load()
        self.q_norm = self.uq = None             # low-rank query only
        self.kv_norm: torch.Tensor = None
        self.w_uk: torch.Tensor = None           # [H, rank, d]: q_nope -> q'
        self.w_ukv: torch.Tensor = None          # [H*d + H*v, rank]: c -> k | v
        self.w_uv: torch.Tensor = None           # [H, v, rank] view of w_ukv
        self.sink = None                         # [H] fp32
        self.cos_sin: torch.Tensor = None

    # ------------------------------------------------------------- weights

    def shapes(self) -> List[Tuple[str, Tuple[int, ...]]]:
        """Checkpoint tensors of the whole (unsharded) mixer."""
        s, w = self.spec, self.width
        qk = s.heads * (s.dim + s.rot_dim)
        if s.q_rank:
            out = [("dq", (s.q_rank, w)), ("dq.norm", (s.q_rank,)), ("uq", (qk, s.q_rank))]
        else:
            out = [("q", (qk, w))]
        out += [
            ("dkv", (s.kv_rank + s.rot_dim, w)), ("dkv.norm", (s.kv_rank,)),
            ("uk", (s.heads * s.dim, s.kv_rank)), ("uv", (s.heads * s.vdim, s.kv_rank)),
        ]
        if s.head_gate:
            out.append(("g", (s.heads, w)))
        if s.sink:
            out.append(("sink", (s.heads,)))
        return out + [("o", (w, s.heads * s.vdim))]

    def _mine(self, t: torch.Tensor, per_head: int) -> torch.Tensor:
        """This rank's heads of a [heads * per_head, k] tensor."""
        return t[self.head0 * per_head : (self.head0 + self.heads) * per_head]

    def _pad_query(self, t: torch.Tensor) -> torch.Tensor:
        s, k = self.spec, t.shape[1]
        t = self._mine(t, s.dim + s.rot_dim).view(self.heads, s.dim + s.rot_dim, k)
        rot = t[:, s.dim :]
        if s.rope_half:
            rot = pair_halves(rot, s.rot_dim, 1)
        out = t.new_zeros(self.heads, self.d + self.rot, k)
        out[:, : s.dim] = t[:, : s.dim]
        out[:, self.d : self.d + s.rot_dim] = rot
        return out.view(self.q_dim, k)

    def _unpad_query(self, t: torch.Tensor) -> torch.Tensor:
        s = self.spec
        t = t.view(self.heads, self.d + self.rot, t.shape[1])
        rot = t[:, self.d : self.d + s.rot_dim]
        if s.rope_half:
            rot = unpair_halves(rot, s.rot_dim, 1)
        t = torch.cat([t[:, : s.dim], rot], 1)
        return t.reshape(-1, t.shape[2])

    def _shared_key(self, dkv: torch.Tensor, reorder) -> torch.Tensor:
        """dkv with its rotated rows reordered."""
        if not self.spec.rope_half:
            return dkv
        rank = self.spec.kv_rank
        return torch.cat([dkv[:rank], reorder(dkv[rank:], self.spec.rot_dim, 0)])

    def load(self, get: Get, p: str) -> Dict[str, torch.Tensor]:
        """Install the mixer's own weights; returns its rows of the layer's
        input projection ("q", "kv", "gate") and columns of the output
        projection ("o")."""
        s, H = self.spec, self.heads
        sections: Dict[str, torch.Tensor] = {}
        if s.q_rank:
            sections["q"] = pad_to(get(p + "dq"), self.q_rank, self.width)
            self.q_norm = pad_to(get(p + "dq.norm"), self.q_rank)
            uq = self._pad_query(get(p + "uq"))
            self.uq = pad_to(uq, uq.shape[0], self.q_rank)
        else:
            sections["q"] = self._pad_query(get(p + "q"))
        sections["kv"] = self._shared_key(get(p + "dkv"), pair_halves)
        if s.head_gate:
            sections["gate"] = self._mine(get(p + "g"), 1)
        if s.sink:
            self.sink = self._mine(get(p + "sink"), 1).float().contiguous()
        self.kv_norm = get(p + "dkv.norm").contiguous()
        uk = self._mine(get(p + "uk"), s.dim).view(H, s.dim, s.kv_rank)
        uv = self._mine(get(p + "uv"), s.vdim).view(H, s.vdim, s.kv_rank)
        self.w_uk = pad_to(uk.transpose(1, 2), H, self.rank, self.d).contiguous()
        self.w_ukv = torch.cat([
            pad_to(uk, H, self.d, self.rank).reshape(H * self.d, self.rank),
            pad_to(uv, H, self.v, self.rank).reshape(H * self.v, self.rank),
        ])
        self.w_uv = self.w_ukv[H * self.d :].view(H, self.v, self.rank)
        o = get(p + "o")
        o = o.view(self.width, s.heads, s.vdim)[:, self.head0 : self.head0 + H]
        sections["o"] = pad_to(o, self.width, H, self.v).reshape(self.width, self.out_dim)
        return sections

    def export(self, sections: Dict[str, torch.Tensor], p: str) -> Dict[str, torch.Tensor]:
        """Inverse of load() (unsharded models)."""
        s, H = self.spec, self.heads
        out = {}
        if s.q_rank:
            out[p + "dq"] = sections["q"][: s.q_rank]
            out[p + "dq.norm"] = self.q_norm[: s.q_rank]
            out[p + "uq"] = self._unpad_query(self.uq)[:, : s.q_rank]
        else:
            out[p + "q"] = self._unpad_query(sections["q"])
        out[p + "dkv"] = self._shared_key(sections["kv"], unpair_halves)
        out[p + "dkv.norm"] = self.kv_norm
        k = self.w_ukv[: H * self.d].view(H, self.d, self.rank)
        out[p + "uk"] = k[:, : s.dim, : s.kv_rank].reshape(H * s.dim, s.kv_rank)
        out[p + "uv"] = self.w_uv[:, : s.vdim, : s.kv_rank].reshape(H * s.vdim, s.kv_rank)
        if s.head_gate:
            out[p + "g"] = sections["gate"]
        if s.sink:
            out[p + "sink"] = self.sink.to(self.w_uk.dtype)
        o = sections["o"].view(self.width, H, self.v)[:, :, : s.vdim]
        out[p + "o"] = o.reshape(self.width, H * s.vdim)
        return out

    # --------------------------------------------------------------- cache

    def new_cache(self, num_blocks: int, block_size: int, dtype, device) -> torch.Tensor:
        # uninitialised: a row is written before any query can see it
        return torch.empty(num_blocks, block_size, self.row, dtype=dtype, device=device)

    # ------------------------------------------------------------- forward

    def forward(self, q: torch.Tensor, kv: torch.Tensor, gate, batch: FlatBatch,
                cache: torch.Tensor, out: torch.Tensor) -> None:
        """q, kv, gate: the sections of the fused projection (row-strided
        views); writes out [N, out_dim] (row-strided view)."""
        s, H, N = self.spec, self.heads, q.shape[0]
        low_rank = (q, self.q_norm, s.q_rank) if s.q_rank else ()
        cq = ops.latent_inputs(
            kv, self.kv_norm, self.eps, s.kv_rank, s.rot_dim, self.rank,
            batch.positions, batch.slot_mapping, self.cos_sin, cache, *low_rank,
        )
        if s.q_rank:
            q = ops.linear(cq, self.uq)
        q = q.as_strided((N, H, self.d + self.rot), (q.stride(0), self.d + self.rot, 1))
        out = out.as_strided((N, H, self.v), (out.stride(0), self.v, 1))
        expanded, row0 = batch.memo(
            ("latent_split", s.window, self.rank, self.d, self.v), lambda: self._split(q, batch)
        )
        if row0 < N:
            qa = torch.empty(N - row0, H, self.rank, dtype=q.dtype, device=q.device)
            ops.head_linear(q[row0:, :, : self.d], self.w_uk, qa)
            latent = ops.latent_attention(
                qa, q[row0:, :, self.d :], self.cos_sin, s.rot_dim, cache, batch, s.scale,
                s.window, row0, expanded, self.sink,
            )
            ops.head_linear(latent, self.w_uv, out[row0:], None if gate is None else gate[row0:])
        if expanded:  # after: the rows above may include expanded chunks'
            ops.latent_expanded_prefill(
                q, self.w_ukv, gate, self.cos_sin, s.rot_dim, cache, batch, expanded,
                self.rank, s.scale, s.window, out, self.sink,
            )

    def _split(self, q: torch.Tensor, batch: FlatBatch) -> Tuple[Tuple[int, ...], int]:
        """The prefill chunks to run expanded, by products per head and chunk,
        and the first row that is not in one of the leading ones."""
        if not batch.prefills or not ops.can_expand(q, self.d, self.v, self.rot):
            return (), 0
        window = self.spec.window or 1 << 30
        per_expansion = self.rank * (self.d + self.v)
        chunks = []
        for i, m in enumerate(batch.prefills):
            seen = m.query_len * min(window, m.ctx_len + (m.query_len + 1) // 2)
            keys = m.seq_len - max(0, m.ctx_len - window + 1)
            expanded = keys * per_expansion + seen * (self.d + self.rot + self.v)
            absorbed = m.query_len * per_expansion + seen * (2 * self.rank + self.rot)
            if expanded <= absorbed:
                chunks.append(i)
        row0 = 0
        for i, m in enumerate(batch.prefills):
            if i not in chunks:
                break
            row0 += m.query_len
        return tuple(chunks), row0
