"""Lobuvik: attention and a feed-forward side by side, each on a layer norm of its own.

    x = scale * embed[token]
    layer:  x <- x + (mixer(norm1(x)) + ff(norm2(x)))
    logits = head . norm(x)

The mixers are grouped attention with sigmoid weights, distance biases and short
convolutions, latent attention with a window and a sink, and rotated grouped attention
with a window, capped scores and head gates.  The feed-forward is dense or a mixture
of experts with a shared one.

Execution.  The residual is fp32.  Both norms of a layer share their statistics, so one
pass over x adds the last layer's results and writes both inputs of the next.  The
mixer's heads and the dense (or shared) GLU meet in one output projection, whose fp32
accumulation does their sum; the routed experts' rows join in the residual update.

Attention layers have pages; those with short convolutions also have a state slot per
sequence that holds the last projected values.

Tensor parallelism: heads and feed-forward columns are sharded, routers replicated; one
all-reduce per layer.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import torch

from .. import ops
from ..engine.batch import FlatBatch
from ..engine.config import EngineConfig, ExpertsSpec, LatentAttentionSpec, LayerSpec, ModelConfig
from .experts import Experts
from .grouped_attention import GroupedAttention
from .latent_attention import LatentAttention
from .layout import Get, fuse_columns, pad_to, round_up, stack_rows, summed_linear
from .llama import _dtype_of
from .rotary import rotation_table


class LobuvikLayer:
    def __init__(self, spec: LayerSpec, cfg: ModelConfig, tp_rank: int, tp_world: int):
        self.width, self.tp_rank = cfg.hidden_size, tp_rank
        self.latent = isinstance(spec.mixer, LatentAttentionSpec)
        kind = LatentAttention if self.latent else GroupedAttention
        self.mixer = kind(spec.mixer, self.width, cfg.rms_eps, tp_rank, tp_world)
        self.mlp = spec.mlp
        self.experts: Optional[Experts] = None
        #: the GLU every token runs: the dense feed-forward or the shared expert
        self.glu, self.glu_at = spec.mlp, "mlp."
        if isinstance(spec.mlp, ExpertsSpec):
            self.experts = Experts(spec.mlp, self.width, tp_rank, tp_world)
            self.glu, self.glu_at = spec.mlp.shared, "mlp.shared."
        self.ff = self.ff_pad = 0
        if self.glu:
            if self.glu.width % tp_world:
                raise ValueError("TP degree must divide the feed-forward width")
            self.ff = self.glu.width // tp_world
            self.ff_pad = round_up(self.ff, 16)
        self.norm1: torch.Tensor = None
        self.norm2: Optional[torch.Tensor] = None     # no feed-forward: None
        # latent attention: its fused input projection
        self.w_in: Optional[torch.Tensor] = None
        self.sections: Dict[str, Tuple[int, int]] = {}
        self.gate_up: Optional[torch.Tensor] = None
        # output projections over column ranges of [heads | GLU], summed
        self.w_out: List[torch.Tensor] = []

    # ------------------------------------------------------------- weights

    def shapes(self) -> List[Tuple[str, Tuple[int, ...]]]:
        w = self.width
        out = [("norm1", (w,))] + [("mix." + n, s) for n, s in self.mixer.shapes()]
        if self.mlp:
            out.append(("norm2", (w,)))
        if self.experts:
            out += [("mlp." + n, s) for n, s in self.experts.shapes()]
        if self.glu:
            ff, p = self.glu.width, self.glu_at
            out += [(p + "gate", (ff, w)), (p + "up", (ff, w)), (p + "down", (w, ff))]
        return out

    def load(self, get: Get, p: str) -> None:
        self.norm1 = get(p + "norm1")
        if self.latent:
            sec = self.mixer.load(get, p + "mix.")
            outs = [sec.pop("o")]
            self.w_in, self.sections = stack_rows(list(sec.items()), self.width)
        else:
            self.mixer.load(get, p + "mix.")
            outs = [self.mixer.w_out]
        if self.mlp:
            self.norm2 = get(p + "norm2")
        if self.experts:
            self.experts.load(get, p + "mlp.")
        if self.glu:
            mine = slice(self.tp_rank * self.ff, (self.tp_rank + 1) * self.ff)
            q = p + self.glu_at
            self.gate_up = torch.cat([
                pad_to(get(q + n)[mine], self.ff_pad, self.width) for n in ("gate", "up")
            ])
            outs.append(pad_to(get(q + "down")[:, mine], self.width, self.ff_pad))
        self.w_out = fuse_columns(outs)
        if not self.latent:  # a view, not a second copy
            self.mixer.w_out = self.w_out[0][:, : self.mixer.out_dim]

    def export(self, p: str) -> Dict[str, torch.Tensor]:
        m, w_out = self.mixer, torch.cat(self.w_out, 1)
        out = {p + "norm1": self.norm1}
        if self.latent:
            sec = {n: self.w_in[at : at + rows] for n, (at, rows) in self.sections.items()}
            sec["o"] = w_out[:, : m.out_dim].contiguous()
            out.update(m.export(sec, p + "mix."))
        else:
            m.w_out = w_out[:, : m.out_dim].contiguous()
            out.update(m.export(p + "mix."))
        if self.mlp:
            out[p + "norm2"] = self.norm2
        if self.experts:
            out.update(self.experts.export(p + "mlp."))
        if self.glu:
            q = p + self.glu_at
            out[q + "gate"] = self.gate_up[: self.ff]
            out[q + "up"] = self.gate_up[self.ff_pad : self.ff_pad + self.ff]
            out[q + "down"] = w_out[:, m.out_dim : m.out_dim + self.ff]
        return out

    # ------------------------------------------------------------- forward

    def sublayers(self, h1: torch.Tensor, h2: Optional[torch.Tensor], batch: FlatBatch, cache,
                  ring: Optional[torch.Tensor]):
        """mixer(h1) + ff(h2) without the routed experts, [N, width], and those: rows and
        weights per (token, choice), or None."""
        m, N = self.mixer, h1.shape[0]
        mixed = torch.empty(N, m.out_dim + self.ff_pad, dtype=h1.dtype, device=h1.device)
        routed = self.experts.forward(h2) if self.experts else None
        if self.glu:
            g = self.glu
            ops.clamped_glu(
                ops.linear(h2[:, : self.width], self.gate_up), g.limit, g.alpha, g.offset,
                mixed[:, m.out_dim :], g.cubic,
            )
        heads, bias = mixed[:, : m.out_dim], None
        if self.latent:
            proj = ops.linear(h1, self.w_in)
            q, kv, gate = (
                proj[:, at : at + rows] if rows else None
                for at, rows in (self.sections.get(n, (0, 0)) for n in ("q", "kv", "gate"))
            )
            m.forward(q, kv, gate, batch, cache, heads)
        else:
            m.attend(h1, batch, cache, ring, heads)
            bias = m.out_bias
        return summed_linear(mixed, self.w_out, bias), routed


class LobuvikForCausalLM:
    def __init__(self, cfg: ModelConfig, ecfg: EngineConfig, device: str,
                 tp_rank: int = 0, tp_world: int = 1):
        self.cfg = cfg
        self.ecfg = ecfg
        self.device = torch.device(device)
        self.dtype = _dtype_of(cfg)
        self.tp_rank = tp_rank
        self.tp_world = tp_world
        self.layers: List[LobuvikLayer] = [
            LobuvikLayer(s, cfg, tp_rank, tp_world) for s in cfg.layers
        ]
        self._install_rotations()
        self.embed: Optional[torch.Tensor] = None
        self.head: Optional[torch.Tensor] = None
        self.final_norm: Optional[torch.Tensor] = None
        # per layer: keys and values, or latent rows; convolution inputs, if any
        self.pages: List = [None] * len(self.layers)
        self.rings: List[Optional[torch.Tensor]] = [None] * len(self.layers)
        # TP all-reduce hook installed by the engine
        self.all_reduce = None

    def _install_rotations(self) -> None:
        """One table per distinct rotation; a speculative step may run one position past
        the limit."""
        positions = min(self.ecfg.max_model_len, self.cfg.max_position) + 1
        tables: Dict[tuple, torch.Tensor] = {}
        for layer in self.layers:
            s = layer.mixer.spec
            if layer.latent:
                key = (s.rope_base, s.rot_dim, s.rope_scaling)
            elif s.rotary:
                key = (s.rotary.base, s.rotary.dims, s.rotary.scaling)
            else:
                continue
            if key not in tables:
                tables[key] = rotation_table(positions, *key, self.device)
            layer.mixer.cos_sin = tables[key]

    # ------------------------------------------------------------- weights

    def weight_shapes(self) -> List[Tuple[str, Tuple[int, ...]]]:
        """Checkpoint tensors of the whole model."""
        w, v = self.cfg.hidden_size, self.cfg.vocab_size
        out = [("embed", (v, w)), ("final.norm", (w,)), ("head", (v, w))]
        for i, layer in enumerate(self.layers):
            out += [(f"l{i}." + n, s) for n, s in layer.shapes()]
        return out

    def load_tensors(self, get: Get) -> None:
        """get(name) -> the whole checkpoint tensor; kept in the model's dtype."""
        shapes = dict(self.weight_shapes())

        def mine(name: str) -> torch.Tensor:
            t = get(name)
            if tuple(t.shape) != shapes[name]:
                raise ValueError(f"{name}: shape {tuple(t.shape)}, config says {shapes[name]}")
            return t.to(self.device, self.dtype)

        self.embed, self.head = mine("embed"), mine("head")
        self.final_norm = mine("final.norm")
        for i, layer in enumerate(self.layers):
            layer.load(mine, f"l{i}.")

    def random_init(self, seed: int = 0) -> None:
        """Random weights of the config's shapes.  Every rank draws the same
        whole tensors and keeps its slice, so a TP group holds one model."""
        g = torch.Generator(device=self.device).manual_seed(seed)
        shapes = dict(self.weight_shapes())

        def draw(name: str) -> torch.Tensor:
            t = torch.empty(shapes[name], dtype=self.dtype, device=self.device)
            if name.rsplit(".", 1)[-1] in ("norm", "norm1", "norm2", "temp"):
                return t.fill_(1.0)
            if name.endswith(".pb"):  # few keys weigh much
                return t.fill_(-4.0)
            std = 0.5 if name.endswith(".conv") else 0.02
            return t.normal_(0.0, std, generator=g)

        self.load_tensors(draw)

    def named_tensors(self) -> Dict[str, torch.Tensor]:
        out = {"embed": self.embed, "final.norm": self.final_norm, "head": self.head}
        for i, layer in enumerate(self.layers):
            out.update(layer.export(f"l{i}."))
        return out

    def load_safetensors(self, path: str) -> None:
        from .weights import load_checkpoint

        load_checkpoint(self, path)

    # ----------------------------------------------------- pages and states

    def allocate_kv_cache(self, num_blocks: int, block_size: int) -> None:
        for i, layer in enumerate(self.layers):
            self.pages[i] = layer.mixer.new_cache(num_blocks, block_size, self.dtype, self.device)

    def kv_block_bytes(self, block_size: int) -> int:
        rows = sum(x.mixer.row if x.latent else x.mixer.cache_row for x in self.layers)
        return block_size * rows * self.dtype.itemsize

    @property
    def caches(self) -> List[torch.Tensor]:
        return [t for p in self.pages for t in (p if isinstance(p, tuple) else (p,))]

    def allocate_state(self, num_slots: int) -> None:
        for i, layer in enumerate(self.layers):
            if not layer.latent:
                self.rings[i] = layer.mixer.new_state(num_slots, self.dtype, self.device)

    @property
    def state_slot_bytes(self) -> int:
        """Of one sequence; 0: no layer keeps a state."""
        size = self.dtype.itemsize
        return sum(x.mixer.state_bytes(size) for x in self.layers if not x.latent)

    @property
    def states(self) -> List[torch.Tensor]:
        return [t for t in self.rings if t is not None]

    def step_bytes(self, tokens: int) -> int:
        """What a step of so many tokens holds beyond a dense layer's activations."""
        return max((x.experts.step_bytes(tokens) for x in self.layers if x.experts), default=0)

    # -------------------------------------------------------------- forward

    def _all_reduced(self, y: torch.Tensor, routed):
        """Sum a layer's results over the ranks, the routed experts' first folded in."""
        if routed is not None:
            part = torch.zeros(y.shape, dtype=torch.float32, device=y.device)
            ops.residual_norm(part, y, 0.0, experts=routed)
            y = part.to(y.dtype)
        return self.all_reduce(y)

    def forward(self, batch: FlatBatch, trace: Optional[list] = None) -> torch.Tensor:
        """Logits [len(batch.logit_rows), vocab] fp32; ``trace`` collects the residual
        after every layer."""
        eps, w, N = self.cfg.rms_eps, self.cfg.hidden_size, batch.num_tokens
        x = torch.empty(N, w, dtype=torch.float32, device=self.device)
        ops.embed_positions(
            batch.token_ids, batch.positions, self.embed, None, x, scale=self.cfg.embed_scale
        )
        h1 = torch.empty(N, w, dtype=self.dtype, device=self.device)
        # zero columns up to whole matrix-core steps, for the experts
        w_pad = max((a.experts.in_pad for a in self.layers if a.experts), default=w)
        new = torch.zeros if w_pad > w else torch.empty
        h2 = new(N, w_pad, dtype=self.dtype, device=self.device)

        def residual(y, layer, experts=None):
            if layer is None:
                ops.residual_norm(x, y, eps, experts=experts)
            else:
                ops.residual_norm(
                    x, y, eps, None, layer.norm1, h1, x_norm2=layer.norm2,
                    out2=None if layer.norm2 is None else h2[:, :w], experts=experts,
                )

        residual(None, self.layers[0] if self.layers else None)
        for i, layer in enumerate(self.layers):
            y, routed = layer.sublayers(h1, h2, batch, self.pages[i], self.rings[i])
            if self.all_reduce is not None:
                y, routed = self._all_reduced(y, routed), None
            residual(y, self.layers[i + 1] if i + 1 < len(self.layers) else None, routed)
            if trace is not None:
                trace.append(x.clone())
        h = ops.layernorm(x[batch.logit_rows], self.final_norm, eps, self.dtype)
        return ops.linear(h, self.head).float()
