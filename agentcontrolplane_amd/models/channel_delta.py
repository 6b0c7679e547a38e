"""Gated delta rule with one decay per head and key channel.

    q, k, v = silu(conv(W h));  q, k to unit length per head, q also * dim^-1/2
    beta = sigmoid(W_b h)
    g = exp(-exp(A_log) * softplus(W_a2 W_a1 h + dt_bias))       [heads, dim]
    S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
    out = W_o (rmsnorm(o) * w * sigmoid(W_g2 W_g1 h))

A sequence's state is S [heads, dim, vdim] in fp32 and the convolutions' last inputs
in a ring by position, both in the slot the scheduler gave it (engine/state.py).

One GEMM makes [q | k | v | b | a1 | g1]; the convolution, the recurrence and the
output norm work on its sections in place.
"""
from __future__ import annotations

from typing import Dict, List, Tuple

import torch

from .. import ops
from ..engine.batch import FlatBatch
from ..engine.config import ChannelDeltaSpec
from .layout import Get, pad_to, round_up, stack_rows


class ChannelDelta:
    def __init__(self, spec: ChannelDeltaSpec, width: int, eps: float,
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
        self.w_a2: torch.Tensor = None
        self.w_g2: torch.Tensor = None
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
        return out + [
            ("b", (s.heads, w)), ("A_log", (s.heads,)), ("norm", (s.vdim,)),
            ("a1", (s.decay_rank, w)), ("a2", (s.heads * s.dim, s.decay_rank)),
            ("dt_bias", (s.heads * s.dim,)),
            ("g1", (s.gate_rank, w)), ("g2", (s.heads * s.vdim, s.gate_rank)),
            ("o", (w, s.heads * s.vdim)),
        ]

    def _mine(self, t: torch.Tensor) -> torch.Tensor:
        """This rank's heads of [heads * size, ...]."""
        n = t.shape[0] * self.kv_heads // self.spec.kv_heads
        return t[self.tp_rank * n : (self.tp_rank + 1) * n]

    def load(self, get: Get, p: str) -> None:
        s = self.spec
        names = [n for n, _, _ in self._conv_parts()]
        ra, rg = round_up(s.decay_rank, 16), round_up(s.gate_rank, 16)
        self.w_in, self.sections = stack_rows([
            ("qkv", torch.cat([self._mine(get(p + n)) for n in names])),
            ("b", self._mine(get(p + "b"))),
            ("a1", pad_to(get(p + "a1"), ra, self.width)),
            ("g1", pad_to(get(p + "g1"), rg, self.width)),
        ], self.width)
        self.conv = torch.cat([self._mine(get(p + n + ".conv")) for n in names]).contiguous()
        self.w_a2 = pad_to(self._mine(get(p + "a2")), self.heads * s.dim, ra).contiguous()
        self.w_g2 = pad_to(self._mine(get(p + "g2")), self.heads * s.vdim, rg).contiguous()
        self.A_log = self._mine(get(p + "A_log")).float().contiguous()
        self.dt_bias = self._mine(get(p + "dt_bias")).float().contiguous()
        self.norm = get(p + "norm").float().contiguous()
        self.w_out = self._mine(get(p + "o").t()).t().contiguous()

    def export(self, p: str) -> Dict[str, torch.Tensor]:
        """Inverse of load() (unsharded models)."""
        s, dt, out, at = self.spec, self.w_in.dtype, {}, 0

        def section(name, rows=None):
            start, n = self.sections[name]
            return self.w_in[start : start + (rows or n)]

        for name, heads, size in self._conv_parts():
            out[p + name] = self.w_in[at : at + heads * size]
            out[p + name + ".conv"] = self.conv[at : at + heads * size]
            at += heads * size
        out[p + "b"] = section("b")
        out[p + "A_log"], out[p + "norm"] = self.A_log.to(dt), self.norm.to(dt)
        out[p + "a1"], out[p + "g1"] = section("a1", s.decay_rank), section("g1", s.gate_rank)
        out[p + "a2"] = self.w_a2[:, : s.decay_rank]
        out[p + "g2"] = self.w_g2[:, : s.gate_rank]
        out[p + "dt_bias"], out[p + "o"] = self.dt_bias.to(dt), self.w_out
        return out

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

    def forward(self, h: torch.Tensor, batch: FlatBatch,
                state: Tuple[torch.Tensor, torch.Tensor]) -> torch.Tensor:
        """h [N, width] -> this rank's part of [N, width]."""
        proj = ops.linear(h, self.w_in)

        def section(name):
            at, rows = self.sections[name]
            return proj[:, at : at + rows]

        z = ops.linear(section("a1"), self.w_a2)
        gate = ops.linear(section("g1"), self.w_g2)
        out = ops.channel_delta(
            section("qkv"), self.conv, section("b"), z, self.A_log, self.dt_bias, gate,
            self.norm, self.eps, self.spec.unit_eps, self.kv_heads, *state, batch,
        )
        return ops.linear(out, self.w_out)
