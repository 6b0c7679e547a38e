"""Gated delta rule with one decay per head and key channel, or one per head.

    q, k, v = silu(conv(W h));  q, k to unit length per head, q also * dim^-1/2
    beta = sigmoid(W_b h)
    g = exp(-exp(A_log) * softplus(W_a h + dt_bias))       [heads, dim] or [heads]
    S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
    out = W_o (rmsnorm(o) * w * gate(W_g h)),  gate sigmoid or silu

W_a and W_g may be products of two (low rank): W_a2 W_a1, W_g2 W_g1.

A sequence's state is S [heads, dim, vdim] in fp32 and the convolutions' last inputs
in a ring by position, both in the slot the scheduler gave it (engine/state.py).

One GEMM makes [q | k | v | b | a or a1 | g or g1], and whatever else a layer wants
from the same input; the convolution, the recurrence and the output norm work on its
sections in place.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import torch

from .. import ops
from ..engine.batch import FlatBatch
from ..engine.config import GatedDeltaSpec
from .layout import Get, pad_to, round_up, section_bias, stack_rows


class GatedDelta:
    def __init__(self, spec: GatedDeltaSpec, width: int, eps: float,
                 tp_rank: int, tp_world: int):
        if spec.heads % spec.kv_heads:
            raise ValueError("kv_heads must divide heads")
        if spec.kv_heads % tp_world:
            raise ValueError("TP degree must divide the key head count")
        self.spec, self.width, self.eps = spec, width, eps
        self.heads, self.kv_heads = spec.heads // tp_world, spec.kv_heads // tp_world
        self.tp_rank = tp_rank
        #: convolved channels: q | k | v
        self.channels = 2 * self.kv_heads * spec.dim + self.heads * spec.vdim
        self.w_in: torch.Tensor = None
        self.sections: Dict[str, Tuple[int, int]] = {}
        self.conv: torch.Tensor = None     # [channels, taps]
        self.bias: Optional[torch.Tensor] = None
        self.w_a2: Optional[torch.Tensor] = None
        self.w_g2: Optional[torch.Tensor] = None
        self.w_out: torch.Tensor = None
        # fp32
        self.A_log = self.dt_bias = self.norm = None

    # ------------------------------------------------------------- weights

    def _conv_parts(self) -> List[Tuple[str, int, int]]:
        """(tensor, heads of the whole model, head size)"""
        s = self.spec
        return [("q", s.kv_heads, s.dim), ("k", s.kv_heads, s.dim), ("v", s.heads, s.vdim)]

    def shapes(self) -> List[Tuple[str, Tuple[int, ...]]]:
        """Checkpoint tensors of the whole (unsharded) mixer."""
        s, w, out = self.spec, self.width, []
        for name, heads, size in self._conv_parts():
            out += [(name, (heads * size, w)), (name + ".conv", (heads * size, s.conv))]
        out += [("b", (s.heads, w)), ("A_log", (s.heads,)), ("norm", (s.vdim,))]
        for name, rank, rows in self._projections():
            out += [(name + "1", (rank, w)), (name + "2", (rows, rank))] if rank else [
                (name, (rows, w))]
        return out + [("dt_bias", (s.decays,)), ("o", (w, s.heads * s.vdim))]

    def _projections(self) -> List[Tuple[str, int, int]]:
        """(tensor, its inner size or 0, rows of the whole model)"""
        s = self.spec
        return [("a", s.decay_rank, s.decays), ("g", s.gate_rank, s.heads * s.vdim)]

    def _mine(self, t: torch.Tensor) -> torch.Tensor:
        """This rank's heads of [heads * size, ...]."""
        n = t.shape[0] * self.kv_heads // self.spec.kv_heads
        return t[self.tp_rank * n : (self.tp_rank + 1) * n]

    def load(self, get: Get, p: str,
             beside: Optional[Tuple[torch.Tensor, torch.Tensor]] = None) -> None:
        """``beside``: rows and bias of another product of the same input."""
        names = [n for n, _, _ in self._conv_parts()]
        sections = [
            ("qkv", torch.cat([self._mine(get(p + n)) for n in names])),
            ("b", self._mine(get(p + "b"))),
        ]
        second = []
        for name, rank, rows in self._projections():
            if rank:
                r = round_up(rank, 16)
                sections.append((name, pad_to(get(f"{p}{name}1"), r, self.width)))
                w2 = self._mine(get(f"{p}{name}2"))
                second.append(pad_to(w2, w2.shape[0], r).contiguous())
            else:
                sections.append((name, self._mine(get(p + name))))
                second.append(None)
        self.w_a2, self.w_g2 = second
        if beside:
            sections.append(("beside", beside[0]))
        self.w_in, self.sections = stack_rows(sections, self.width)
        if beside:
            self.bias = section_bias(self.w_in, self.sections, {"beside": beside[1]})
        self.conv = torch.cat([self._mine(get(p + n + ".conv")) for n in names]).contiguous()
        self.A_log = self._mine(get(p + "A_log")).float().contiguous()
        self.dt_bias = self._mine(get(p + "dt_bias")).float().contiguous()
        self.norm = get(p + "norm").float().contiguous()
        self.w_out = self._mine(get(p + "o").t()).t().contiguous()

    def export(self, p: str) -> Dict[str, torch.Tensor]:
        """Inverse of load() (unsharded models)."""
        dt, out, at = self.w_in.dtype, {}, 0

        def section(name, rows=None):
            start, n = self.sections[name]
            return self.w_in[start : start + (rows or n)]

        for name, heads, size in self._conv_parts():
            out[p + name] = self.w_in[at : at + heads * size]
            out[p + name + ".conv"] = self.conv[at : at + heads * size]
            at += heads * size
        out[p + "b"] = section("b")
        out[p + "A_log"], out[p + "norm"] = self.A_log.to(dt), self.norm.to(dt)
        for (name, rank, _), second in zip(self._projections(), (self.w_a2, self.w_g2)):
            if rank:
                out[f"{p}{name}1"], out[f"{p}{name}2"] = section(name, rank), second[:, :rank]
            else:
                out[p + name] = section(name)
        out[p + "dt_bias"], out[p + "o"] = self.dt_bias.to(dt), self.w_out
        return out

    def beside(self) -> Tuple[torch.Tensor, torch.Tensor]:
        at, rows = self.sections["beside"]
        return self.w_in[at : at + rows], self.bias[at : at + rows]

    # --------------------------------------------------------------- state

    def new_state(self, num_slots: int, dtype, device) -> Tuple[torch.Tensor, torch.Tensor]:
        """(S, convolution inputs) per slot; uninitialised: a sequence's first
        chunk starts from zero."""
        s = self.spec
        return (
            torch.empty(num_slots, self.heads, s.dim, s.vdim, dtype=torch.float32, device=device),
            torch.empty(num_slots, s.conv, self.channels, dtype=dtype, device=device),
        )

    def state_bytes(self, itemsize: int) -> int:
        s = self.spec
        return 4 * self.heads * s.dim * s.vdim + s.conv * self.channels * itemsize

    # ------------------------------------------------------------- forward

    def mix(self, h: torch.Tensor, batch: FlatBatch, state: Tuple[torch.Tensor, torch.Tensor]):
        """h [N, width] -> the heads ahead of W_o [N, heads * vdim] and, if there is one,
        the product beside the mixer's."""
        proj = ops.linear(h, self.w_in, self.bias)

        def section(name, second=None):
            at, rows = self.sections[name]
            x = proj[:, at : at + rows]
            return x if second is None else ops.linear(x, second)

        out = ops.gated_delta(
            section("qkv"), self.conv, section("b"), section("a", self.w_a2), self.A_log,
            self.dt_bias, section("g", self.w_g2), self.norm, self.eps, self.spec.unit_eps,
            self.kv_heads, *state, batch, gate_silu=self.spec.gate_silu,
        )
        return out, section("beside") if "beside" in self.sections else None

    def forward(self, h: torch.Tensor, batch: FlatBatch,
                state: Tuple[torch.Tensor, torch.Tensor]) -> torch.Tensor:
        """h [N, width] -> this rank's part of [N, width]."""
        return ops.linear(self.mix(h, batch, state)[0], self.w_out)
