"""Tezinex: delta layers and windowed attention layers, sandwich norms, and a learned
average over the depth.

    X_0 = embed[token] + sinusoid(position);  x = X_0
    layer i:  x <- x + m norm(mixer(norm(x)));  x <- x + m norm(ff(norm(x)))
              X_{i+1} = x;  x <- sum_j c_ij X_j
    logits = cap(embed . norm(x))

The norms are RMS norms whose weight is stored as its distance from one.

Execution.  The residual and the states X_j are fp32; the X_j of a step live in one
buffer.  Between two GEMMs of a sublayer pair everything on the residual is one
pass: the sublayer's norm, the addition, storing X_{i+1} and averaging the depth
at a layer's end, and the next sublayer's norm.

Attention layers have pages, delta layers have state slots.  An attention layer may
use an earlier one's keys and values: it then has no cache of its own.

Tensor parallelism: heads and feed-forward columns are sharded, low-rank inner
projections replicated; one all-reduce per sublayer, before its output norm.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import torch

from .. import ops
from ..engine.batch import FlatBatch
from ..engine.config import EngineConfig, GatedDeltaSpec, LayerSpec, ModelConfig
from ..ops.reference import build_cos_sin
from .gated_delta import GatedDelta
from .grouped_attention import GroupedAttention
from .layout import Get, pad_to, round_up
from .llama import _dtype_of

#: norm weights are stored as their distance from this
_NORM_OFFSET = 1.0


class TezinexLayer:
    def __init__(self, spec: LayerSpec, cfg: ModelConfig, tp_rank: int, tp_world: int):
        self.width = cfg.hidden_size
        self.recurrent = isinstance(spec.mixer, GatedDeltaSpec)
        if self.recurrent:
            self.mixer = GatedDelta(spec.mixer, self.width, cfg.rms_eps, tp_rank, tp_world)
        else:
            self.mixer = GroupedAttention(
                spec.mixer, self.width, cfg.rms_eps, tp_rank, tp_world
            )
        self.mlp = spec.mlp
        self.tp_rank = tp_rank
        if self.mlp:
            if self.mlp.width % tp_world:
                raise ValueError("TP degree must divide the feed-forward width")
            self.ff = self.mlp.width // tp_world
            self.ff_pad = round_up(self.ff, 16)
        # norms in and out of the mixer and the feed-forward
        self.norm1 = self.norm1b = self.norm2 = self.norm2b = None
        self.gate_up: torch.Tensor = None
        self.down: torch.Tensor = None
        self.depth: Optional[torch.Tensor] = None   # depth weights, one per state so far

    def shapes(self, index: int, depth_average: bool) -> List[Tuple[str, Tuple[int, ...]]]:
        w = self.width
        out = [("norm1", (w,)), ("norm1b", (w,))]
        out += [("mix." + n, s) for n, s in self.mixer.shapes()]
        if self.mlp:
            ff = self.mlp.width
            out += [("norm2", (w,)), ("norm2b", (w,)), ("mlp.gate", (ff, w)),
                    ("mlp.up", (ff, w)), ("mlp.down", (w, ff))]
        if depth_average:
            out.append(("dwa", (index + 2,)))
        return out

    def load(self, get: Get, p: str, depth_average: bool) -> None:
        self.norm1, self.norm1b = get(p + "norm1"), get(p + "norm1b")
        self.mixer.load(get, p + "mix.")
        if self.mlp:
            self.norm2, self.norm2b = get(p + "norm2"), get(p + "norm2b")
            mine = slice(self.tp_rank * self.ff, (self.tp_rank + 1) * self.ff)
            self.gate_up = torch.cat([
                pad_to(get(p + "mlp." + n)[mine], self.ff_pad, self.width)
                for n in ("gate", "up")
            ])
            self.down = pad_to(get(p + "mlp.down")[:, mine], self.width, self.ff_pad).contiguous()
        if depth_average:
            self.depth = get(p + "dwa")

    def export(self, p: str) -> Dict[str, torch.Tensor]:
        out = {p + "norm1": self.norm1, p + "norm1b": self.norm1b}
        out.update(self.mixer.export(p + "mix."))
        if self.mlp:
            out[p + "norm2"], out[p + "norm2b"] = self.norm2, self.norm2b
            out[p + "mlp.gate"] = self.gate_up[: self.ff]
            out[p + "mlp.up"] = self.gate_up[self.ff_pad : self.ff_pad + self.ff]
            out[p + "mlp.down"] = self.down[:, : self.ff]
        if self.depth is not None:
            out[p + "dwa"] = self.depth
        return out

    def feed_forward(self, h: torch.Tensor) -> torch.Tensor:
        gate_up = ops.linear(h, self.gate_up)
        act = torch.empty(h.shape[0], self.ff_pad, dtype=h.dtype, device=h.device)
        ops.clamped_glu(gate_up, self.mlp.limit, self.mlp.alpha, self.mlp.offset, act)
        return ops.linear(act, self.down)


class TezinexForCausalLM:
    def __init__(self, cfg: ModelConfig, ecfg: EngineConfig, device: str,
                 tp_rank: int = 0, tp_world: int = 1):
        self.cfg = cfg
        self.ecfg = ecfg
        self.device = torch.device(device)
        self.dtype = _dtype_of(cfg)
        self.tp_rank = tp_rank
        self.tp_world = tp_world
        self.layers: List[TezinexLayer] = [
            TezinexLayer(s, cfg, tp_rank, tp_world) for s in cfg.layers
        ]
        self.pos_table: Optional[torch.Tensor] = None
        if cfg.position_base is not None:
            # a speculative step may run one position past the limit
            positions = min(ecfg.max_model_len, cfg.max_position) + 1
            self.pos_table = build_cos_sin(
                positions, cfg.hidden_size, cfg.position_base, self.device, exact=True
            )
        self.embed: Optional[torch.Tensor] = None
        self.final_norm: Optional[torch.Tensor] = None
        self.depth_coef: Optional[torch.Tensor] = None  # [layers, layers + 1] fp32
        # per layer: (keys, values), the owner's for borrowed ones, or (S, conv inputs)
        self.stores: List[Tuple[torch.Tensor, torch.Tensor]] = [None] * len(self.layers)
        # TP all-reduce hook installed by the engine
        self.all_reduce = None

    # ------------------------------------------------------------- weights

    def weight_shapes(self) -> List[Tuple[str, Tuple[int, ...]]]:
        """Checkpoint tensors of the whole model."""
        w = self.cfg.hidden_size
        out = [("embed", (self.cfg.vocab_size, w)), ("final.norm", (w,))]
        for i, layer in enumerate(self.layers):
            out += [(f"l{i}." + n, s) for n, s in layer.shapes(i, self.cfg.depth_average)]
        return out

    def load_tensors(self, get: Get) -> None:
        """get(name) -> the whole checkpoint tensor; kept in the model's dtype."""
        shapes = dict(self.weight_shapes())

        def mine(name: str) -> torch.Tensor:
            t = get(name)
            if tuple(t.shape) != shapes[name]:
                raise ValueError(f"{name}: shape {tuple(t.shape)}, config says {shapes[name]}")
            return t.to(self.device, self.dtype)

        self.embed = mine("embed")
        self.final_norm = mine("final.norm")
        for i, layer in enumerate(self.layers):
            layer.load(mine, f"l{i}.", self.cfg.depth_average)
        if self.cfg.depth_average:
            n = len(self.layers)
            self.depth_coef = torch.zeros(n, n + 1, dtype=torch.float32, device=self.device)
            for i, layer in enumerate(self.layers):
                self.depth_coef[i, : i + 2] = layer.depth.float()

    def random_init(self, seed: int = 0) -> None:
        """Random weights of the config's shapes.  Every rank draws the same
        whole tensors and keeps its slice, so a TP group holds one model."""
        g = torch.Generator(device=self.device).manual_seed(seed)
        shapes = dict(self.weight_shapes())

        def draw(name: str) -> torch.Tensor:
            t = torch.empty(shapes[name], dtype=self.dtype, device=self.device)
            if name.endswith(".mix.norm"):
                return t.fill_(1.0)
            if name.endswith(".dwa"):  # mostly the layer's own result
                t.fill_(0.1)[-1] = 1.0
                return t
            std = 0.5 if name.endswith(".conv") else 0.02
            return t.normal_(0.0, std, generator=g)

        self.load_tensors(draw)

    def named_tensors(self) -> Dict[str, torch.Tensor]:
        out = {"embed": self.embed, "final.norm": self.final_norm}
        for i, layer in enumerate(self.layers):
            out.update(layer.export(f"l{i}."))
        return out

    def load_safetensors(self, path: str) -> None:
        from .weights import load_checkpoint

        load_checkpoint(self, path)

    # ----------------------------------------------------- pages and states

    def allocate_kv_cache(self, num_blocks: int, block_size: int) -> None:
        for i, layer in enumerate(self.layers):
            if layer.recurrent:
                continue
            owner = layer.mixer.spec.kv_from
            self.stores[i] = (
                layer.mixer.new_cache(num_blocks, block_size, self.dtype, self.device)
                if owner is None else self.stores[owner]
            )

    def kv_block_bytes(self, block_size: int) -> int:
        rows = sum(x.mixer.cache_row for x in self.layers if not x.recurrent)
        return block_size * rows * self.dtype.itemsize

    @property
    def caches(self) -> List[torch.Tensor]:
        return [
            t for layer, store in zip(self.layers, self.stores)
            if not layer.recurrent and layer.mixer.spec.kv_from is None for t in store
        ]

    def allocate_state(self, num_slots: int) -> None:
        for i, layer in enumerate(self.layers):
            if layer.recurrent:
                self.stores[i] = layer.mixer.new_state(num_slots, self.dtype, self.device)

    @property
    def state_slot_bytes(self) -> int:
        """Of one sequence; 0: no layer keeps a state."""
        return sum(x.mixer.state_bytes(self.dtype.itemsize) for x in self.layers if x.recurrent)

    @property
    def states(self) -> List[torch.Tensor]:
        return [
            t for layer, store in zip(self.layers, self.stores) if layer.recurrent for t in store
        ]

    def step_bytes(self, tokens: int) -> int:
        """What a step of so many tokens holds beyond a layer's activations: the
        depth states."""
        planes = len(self.layers) + 1 + ops.DEPTH_AHEAD if self.cfg.depth_average else 0
        return 4 * planes * tokens * self.cfg.hidden_size

    # -------------------------------------------------------------- forward

    def _reduced(self, y: torch.Tensor) -> torch.Tensor:
        return y if self.all_reduce is None else self.all_reduce(y)

    def forward(self, batch: FlatBatch, trace: Optional[list] = None) -> torch.Tensor:
        """Logits [len(batch.logit_rows), vocab] fp32; ``trace`` collects what
        every layer hands on."""
        cfg, eps, w, N = self.cfg, self.cfg.rms_eps, self.cfg.hidden_size, batch.num_tokens
        x = torch.empty(N, w, dtype=torch.float32, device=self.device)
        depth = None if self.depth_coef is None else ops.Depth.new(self.depth_coef, N, w)
        ops.embed_positions(
            batch.token_ids, batch.positions, self.embed, self.pos_table, x,
            None if depth is None else depth.states[0],
        )
        kw = dict(center=False, offset=_NORM_OFFSET, mult=cfg.residual_mult)
        h = torch.empty(N, w, dtype=self.dtype, device=self.device)
        ops.residual_norm(x, None, eps, None, self.layers[0].norm1, h, **kw)
        for i, layer in enumerate(self.layers):
            y = self._reduced(layer.mixer.forward(h, batch, self.stores[i]))
            norm_y = layer.norm1b
            if layer.mlp:
                ops.residual_norm(x, y, eps, norm_y, layer.norm2, h, **kw)
                y = self._reduced(layer.feed_forward(h))
                norm_y = layer.norm2b
            last = i + 1 == len(self.layers)
            ops.residual_norm(
                x, y, eps, norm_y, None if last else self.layers[i + 1].norm1,
                None if last else h, depth=depth, layer=i, **kw,
            )
            if trace is not None:
                trace.append(x.clone())
        x = x[batch.logit_rows]
        h = torch.empty(x.shape, dtype=self.dtype, device=self.device)
        ops.residual_norm(x, None, eps, None, self.final_norm, h, **kw)
        return ops.softcap(ops.linear(h, self.embed), cfg.logit_softcap)
