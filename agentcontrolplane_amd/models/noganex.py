"""Noganex: chunked attention layers whose heads mix their scores, and delta layers with
one decay per head; gated results, normed on their way out; layers that share weights.

    x = embed[token]
    layer:  x <- x + norm1(sigmoid(W_1 x + b_1) * mixer(x))
            x <- x + norm2(sigmoid(W_2 x + b_2) * ff(x))
    logits = scale * head . norm(x)

The norms are RMS norms.  The feed-forward is dense (gelu, with biases) or a mixture of
experts with sigmoid scores and a shared expert; it may be absent.

Execution.  The residual is fp32.  A sublayer reads it in the model's dtype; its gate is
more rows of its first product.  Between two products everything on the residual is one
pass: the routed experts' weighted sum, the gate, the norm, the addition and the next
sublayer's input.

Attention layers have pages, delta layers have state slots, one of each per layer also
where the weights are another layer's.

Tensor parallelism: delta heads and feed-forward columns are sharded, with one all-reduce
per sublayer, before its gate; attention, whose norms and scores need all heads at once,
and the gates are replicated.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import torch

from .. import ops
from ..engine.batch import FlatBatch
from ..engine.config import EngineConfig, ExpertsSpec, GatedDeltaSpec, LayerSpec, ModelConfig
from .experts import Experts
from .gated_delta import GatedDelta
from .grouped_attention import GroupedAttention
from .layout import Get, pad_to, round_up, section_bias, stack_rows
from .llama import _dtype_of
from .rotary import rotation_table


class NoganexLayer:
    def __init__(self, spec: LayerSpec, cfg: ModelConfig, tp_rank: int, tp_world: int):
        self.width, self.tp_rank = cfg.hidden_size, tp_rank
        self.recurrent = isinstance(spec.mixer, GatedDeltaSpec)
        if self.recurrent:
            self.mixer = GatedDelta(spec.mixer, self.width, cfg.rms_eps, tp_rank, tp_world)
        else:
            self.mixer = GroupedAttention(spec.mixer, self.width, cfg.rms_eps, 0, 1)
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
        self.w_in: Optional[torch.Tensor] = None      # [gate | up | residual gate rows, width]
        self.in_bias: Optional[torch.Tensor] = None
        self.sections: Dict[str, Tuple[int, int]] = {}
        self.down: Optional[torch.Tensor] = None
        self.down_bias: Optional[torch.Tensor] = None  # on the first rank

    # ------------------------------------------------------------- weights

    def shapes(self) -> List[Tuple[str, Tuple[int, ...]]]:
        w = self.width
        out = [("norm1", (w,)), ("rg1", (w, w)), ("rg1.b", (w,))]
        out += [("mix." + n, s) for n, s in self.mixer.shapes()]
        if self.mlp:
            out += [("norm2", (w,)), ("rg2", (w, w)), ("rg2.b", (w,))]
        if self.experts:
            out += [("mlp." + n, s) for n, s in self.experts.shapes()]
        if self.glu:
            ff, p = self.glu.width, self.glu_at
            for n, rows, cols in (("gate", ff, w), ("up", ff, w), ("down", w, ff)):
                out.append((p + n, (rows, cols)))
                if self.glu.bias:
                    out.append((p + n + ".b", (rows,)))
        return out

    def load(self, get: Get, p: str) -> None:
        self.norm1 = get(p + "norm1")
        self.mixer.load(get, p + "mix.", (get(p + "rg1"), get(p + "rg1.b")))
        if not self.mlp:
            return
        self.norm2 = get(p + "norm2")
        if self.experts:
            self.experts.load(get, p + "mlp.")
        sections, biases = [], {"rg": get(p + "rg2.b")}
        if self.glu:
            mine = slice(self.tp_rank * self.ff, (self.tp_rank + 1) * self.ff)
            q = p + self.glu_at
            for n in ("gate", "up"):
                sections.append((n, pad_to(get(q + n)[mine], self.ff_pad, self.width)))
                if self.glu.bias:
                    biases[n] = get(f"{q}{n}.b")[mine]
            self.down = pad_to(get(q + "down")[:, mine], self.width, self.ff_pad).contiguous()
            if self.glu.bias and self.tp_rank == 0:
                self.down_bias = get(q + "down.b").contiguous()
        sections.append(("rg", get(p + "rg2")))
        self.w_in, self.sections = stack_rows(sections, self.width)
        self.in_bias = section_bias(self.w_in, self.sections, biases)

    def export(self, p: str) -> Dict[str, torch.Tensor]:
        """Inverse of load() (unsharded models)."""
        out = {p + "norm1": self.norm1, **self.mixer.export(p + "mix.")}
        out[p + "rg1"], out[p + "rg1.b"] = self.mixer.beside()
        if not self.mlp:
            return out
        out[p + "norm2"] = self.norm2
        at, n = self.sections["rg"]
        out[p + "rg2"], out[p + "rg2.b"] = self.w_in[at : at + n], self.in_bias[at : at + n]
        if self.experts:
            out.update(self.experts.export(p + "mlp."))
        if self.glu:
            q = p + self.glu_at
            for n in ("gate", "up"):
                at = self.sections[n][0]
                out[q + n] = self.w_in[at : at + self.ff]
                if self.glu.bias:
                    out[f"{q}{n}.b"] = self.in_bias[at : at + self.ff]
            out[q + "down"] = self.down[:, : self.ff]
            if self.glu.bias:
                out[q + "down.b"] = self.down_bias
        return out

    # ------------------------------------------------------------- forward

    def mix(self, h: torch.Tensor, batch: FlatBatch, store):
        """(this rank's part of the mixer's result, its gate before the sigmoid)"""
        heads, gate = self.mixer.mix(h, batch, store)
        return ops.linear(heads, self.mixer.w_out), gate

    def feed_forward(self, h: torch.Tensor):
        """h [N, experts' padded width] -> (this rank's part of the result without the
        routed experts, its gate, those: rows and weights per (token, choice), or None)."""
        proj = ops.linear(h[:, : self.width], self.w_in, self.in_bias)
        at, n = self.sections["rg"]
        routed = self.experts.forward(h) if self.experts else None
        if self.glu:
            g = self.glu
            act = torch.empty(h.shape[0], self.ff_pad, dtype=h.dtype, device=h.device)
            ops.clamped_glu(
                proj[:, : 2 * self.ff_pad], g.limit, g.alpha, g.offset, act, g.cubic
            )
            y = ops.linear(act, self.down, self.down_bias)
        else:
            y = torch.zeros(h.shape[0], self.width, dtype=h.dtype, device=h.device)
        return y, proj[:, at : at + n], routed


class NoganexForCausalLM:
    def __init__(self, cfg: ModelConfig, ecfg: EngineConfig, device: str,
                 tp_rank: int = 0, tp_world: int = 1):
        self.cfg = cfg
        self.ecfg = ecfg
        self.device = torch.device(device)
        self.dtype = _dtype_of(cfg)
        self.tp_rank = tp_rank
        self.tp_world = tp_world
        # a layer that uses another one's weights is that layer, with a store of its own
        own = {i: NoganexLayer(s, cfg, tp_rank, tp_world)
               for i, s in enumerate(cfg.layers) if s.weights_of is None}
        self.layers: List[NoganexLayer] = [
            own[i if s.weights_of is None else s.weights_of] for i, s in enumerate(cfg.layers)
        ]
        self._install_rotations()
        self.embed: Optional[torch.Tensor] = None
        self.head: Optional[torch.Tensor] = None
        self.final_norm: Optional[torch.Tensor] = None
        # per layer: (keys, values) or (S, convolution inputs)
        self.stores: List[Tuple[torch.Tensor, torch.Tensor]] = [None] * len(self.layers)
        # TP all-reduce hook installed by the engine
        self.all_reduce = None

    def _install_rotations(self) -> None:
        """One table per distinct rotation; a speculative step may run one position past
        the limit."""
        positions = min(self.ecfg.max_model_len, self.cfg.max_position) + 1
        tables: Dict[tuple, torch.Tensor] = {}
        for layer in self.layers:
            if layer.recurrent:
                continue
            r = layer.mixer.spec.rotary
            key = (r.base, r.dims, r.scaling)
            if key not in tables:
                tables[key] = rotation_table(positions, *key, self.device)
            layer.mixer.cos_sin = tables[key]

    # ------------------------------------------------------------- weights

    def _owners(self) -> List[Tuple[str, NoganexLayer]]:
        """(tensor prefix, layer) of the layers that have weights of their own"""
        return [(f"l{i}.", layer) for i, (layer, s) in enumerate(zip(self.layers, self.cfg.layers))
                if s.weights_of is None]

    def weight_shapes(self) -> List[Tuple[str, Tuple[int, ...]]]:
        """Checkpoint tensors of the whole model."""
        w, v = self.cfg.hidden_size, self.cfg.vocab_size
        out = [("embed", (v, w)), ("final.norm", (w,)), ("head", (v, w))]
        for p, layer in self._owners():
            out += [(p + n, s) for n, s in layer.shapes()]
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
        for p, layer in self._owners():
            layer.load(mine, p)

    def random_init(self, seed: int = 0) -> None:
        """Random weights of the config's shapes.  Every rank draws the same
        whole tensors and keeps its slice, so a TP group holds one model."""
        g = torch.Generator(device=self.device).manual_seed(seed)
        shapes = dict(self.weight_shapes())

        def draw(name: str) -> torch.Tensor:
            t = torch.empty(shapes[name], dtype=self.dtype, device=self.device)
            if name.rsplit(".", 1)[-1] in ("norm", "norm1", "norm2"):
                return t.fill_(1.0)
            std = 0.5 if name.endswith(".conv") else 0.02
            t.normal_(0.0, std, generator=g)
            if name.endswith(".talk"):  # mostly a head's own scores
                t += torch.eye(len(t), dtype=t.dtype, device=t.device)
            return t

        self.load_tensors(draw)

    def named_tensors(self) -> Dict[str, torch.Tensor]:
        out = {"embed": self.embed, "final.norm": self.final_norm, "head": self.head}
        for p, layer in self._owners():
            out.update(layer.export(p))
        return out

    def load_safetensors(self, path: str) -> None:
        from .weights import load_checkpoint

        load_checkpoint(self, path)

    # ----------------------------------------------------- pages and states

    def allocate_kv_cache(self, num_blocks: int, block_size: int) -> None:
        for i, layer in enumerate(self.layers):
            if not layer.recurrent:
                self.stores[i] = layer.mixer.new_cache(
                    num_blocks, block_size, self.dtype, self.device
                )

    def kv_block_bytes(self, block_size: int) -> int:
        rows = sum(x.mixer.cache_row for x in self.layers if not x.recurrent)
        return block_size * rows * self.dtype.itemsize

    @property
    def caches(self) -> List[torch.Tensor]:
        return [t for layer, store in zip(self.layers, self.stores) if not layer.recurrent
                for t in store]

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
        return [t for layer, store in zip(self.layers, self.stores) if layer.recurrent
                for t in store]

    def step_bytes(self, tokens: int) -> int:
        """What a step of so many tokens holds beyond a dense layer's activations."""
        return max((x.experts.step_bytes(tokens) for x in self.layers if x.experts), default=0)

    # -------------------------------------------------------------- forward

    def _all_reduced(self, y: torch.Tensor, routed):
        """Sum a sublayer's results over the ranks, the routed experts' first folded in."""
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
        ops.embed_positions(batch.token_ids, batch.positions, self.embed, None, x)
        # zero columns up to whole matrix-core steps, for the experts
        w_pad = max((a.experts.in_pad for a in self.layers if a.experts), default=w)
        new = torch.zeros if w_pad > w else torch.empty
        padded = new(N, w_pad, dtype=self.dtype, device=self.device)
        h = padded[:, :w]
        ops.residual_norm(x, None, eps, out=h)
        for i, layer in enumerate(self.layers):
            y, gate = layer.mix(h, batch, self.stores[i])
            if self.all_reduce is not None and layer.recurrent:
                y = self.all_reduce(y)
            ops.residual_norm(x, y, eps, layer.norm1, out=h, gate=gate)
            if layer.mlp:
                y, gate, routed = layer.feed_forward(padded)
                if self.all_reduce is not None:
                    y, routed = self._all_reduced(y, routed), None
                ops.residual_norm(x, y, eps, layer.norm2, out=h, experts=routed, gate=gate)
            if trace is not None:
                trace.append(x.clone())
        x = x[batch.logit_rows]
        h = torch.empty(x.shape, dtype=self.dtype, device=self.device)
        ops.residual_norm(x, None, eps, None, self.final_norm, h, center=False)
        return ops.linear(h, self.head).float().mul_(self.cfg.logit_scale)
