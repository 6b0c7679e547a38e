"""Mixture of experts: a router, small GLUs of which each token uses some, and an
optional shared GLU that every token uses.

    z = W_router h + b;  the ``top`` largest are chosen, weighted by their softmax
    or s = sigmoid(z);  the ``top`` largest s + correction are chosen, weighted by
       scale * s / sum of the chosen s
    out = sum_chosen weight * W_down act(W_gate h, W_up h)   [+ shared(h)]

Router logits and weights are fp32.  The experts' products run over the step's
(token, choice) pairs grouped by expert on the device, so control flow does not depend
on the routing and decode steps can be captured.  Their results stay one row per
pair; the residual update sums a token's rows with its weights (ops.residual_norm).

The shared GLU is a dense one: the layer stacks it with its other dense products.

Zero padding: the inner sizes of both products are rounded up to whole matrix-core
steps.  Tensor parallelism shards every expert's feed-forward width.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import torch

from .. import ops
from ..engine.config import ExpertsSpec
from .layout import Get, pad_to, round_up

#: inner sizes of the experts' products are multiples of this
INNER = 64


class Experts:
    def __init__(self, spec: ExpertsSpec, width: int, tp_rank: int, tp_world: int):
        if not 0 < spec.top <= spec.experts:
            raise ValueError("top must be between 1 and the number of experts")
        if spec.sigmoid and spec.router_bias or spec.correction and not spec.sigmoid:
            raise ValueError("softmax scores may have a bias, sigmoid ones a correction")
        if spec.expert.bias:
            raise ValueError("routed experts have no biases")
        if spec.expert.width % tp_world:
            raise ValueError("TP degree must divide the experts' width")
        self.spec, self.width, self.tp_rank = spec, width, tp_rank
        self.ff = spec.expert.width // tp_world
        self.ff_pad, self.in_pad = round_up(self.ff, INNER), round_up(width, INNER)
        self.router: torch.Tensor = None                 # [experts, in_pad]
        self.router_bias: Optional[torch.Tensor] = None  # fp32; the correction of sigmoids
        self.gate_up: torch.Tensor = None                # [experts, 2 ff_pad, in_pad]
        self.down: torch.Tensor = None                   # [experts, width, ff_pad]

    @property
    def _bias_name(self) -> Optional[str]:
        s = self.spec
        return "router.b" if s.router_bias else "correction" if s.correction else None

    def shapes(self) -> List[Tuple[str, Tuple[int, ...]]]:
        """Checkpoint tensors of the router and the routed experts."""
        s, w, ff = self.spec, self.width, self.spec.expert.width
        out = [("router", (s.experts, w))]
        if self._bias_name:
            out.append((self._bias_name, (s.experts,)))
        for e in range(s.experts):
            out += [(f"e{e}.gate", (ff, w)), (f"e{e}.up", (ff, w)), (f"e{e}.down", (w, ff))]
        return out

    def load(self, get: Get, p: str) -> None:
        s = self.spec
        mine = slice(self.tp_rank * self.ff, (self.tp_rank + 1) * self.ff)
        router = get(p + "router")
        self.router = pad_to(router, s.experts, self.in_pad).contiguous()
        if self._bias_name:
            self.router_bias = get(p + self._bias_name).float().contiguous()
        self.gate_up = router.new_zeros(s.experts, 2, self.ff_pad, self.in_pad)
        self.down = router.new_zeros(s.experts, self.width, self.ff_pad)
        for e in range(s.experts):
            for n, name in enumerate(("gate", "up")):
                self.gate_up[e, n, : self.ff, : self.width] = get(f"{p}e{e}.{name}")[mine]
            self.down[e, :, : self.ff] = get(f"{p}e{e}.down")[:, mine]
        self.gate_up = self.gate_up.flatten(1, 2)

    def export(self, p: str) -> Dict[str, torch.Tensor]:
        """Inverse of load() (unsharded models)."""
        out = {p + "router": self.router[:, : self.width]}
        if self.router_bias is not None:
            out[p + self._bias_name] = self.router_bias.to(self.router.dtype)
        for e in range(self.spec.experts):
            gate, up = self.gate_up[e].view(2, self.ff_pad, self.in_pad)[:, : self.ff, : self.width]
            out[f"{p}e{e}.gate"], out[f"{p}e{e}.up"] = gate, up
            out[f"{p}e{e}.down"] = self.down[e, :, : self.ff]
        return out

    def step_bytes(self, tokens: int) -> int:
        """Rows per (token, choice) that a step holds."""
        row = (self.ff_pad + self.width) * self.router.element_size() + 16
        return tokens * self.spec.top * row

    def forward(self, h: torch.Tensor) -> Tuple[torch.Tensor, torch.Tensor]:
        """h [N, in_pad] (zero beyond the width) -> this rank's part of every choice's
        result [N, top, width] and its weight [N, top] fp32."""
        s = self.spec
        ids, weights = ops.moe_route(
            h, self.router, self.router_bias, s.top, sigmoid=s.sigmoid, scale=s.scale
        )
        return ops.moe_experts(h, self.gate_up, self.down, ids, s.expert), weights
