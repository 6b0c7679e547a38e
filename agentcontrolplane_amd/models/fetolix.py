"""Fetolix: parallel-block decoder with latent attention, looped layers and a
per-layer token input.

    x0 = embed[token]
    entering each pass of the loop:  x <- W_in [x; x0]
    h  = layernorm(x)
    x <- x + (attention(h) + glu(h))
    y  = W_proj (gelu(W_gate x) * side_embed_i[token]);  x <- x + rmsnorm(y)
    logits = embed . layernorm(x)

Execution.  The residual is fp32.  Both sublayers read h and are summed, so a
layer's large GEMMs are one over [query | latent | head gates | glu gate | glu up]
and one over [attention heads | glu], whose fp32 accumulation does the sum.
The kernels between them work on slices of those buffers in place.  The residual
updates, the side norm and the next layer's input norm are one pass over x.

A looped layer has one cache per pass (ModelConfig.layer_runs); all caches share
the sequence's block table, so the block manager sees one pool.

Tensor parallelism: heads and GLU columns are sharded, latents and the side
input replicated; one all-reduce per layer run, after the output GEMM.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import torch
import torch.nn.functional as F

from .. import ops
from ..engine.batch import FlatBatch
from ..engine.config import EngineConfig, LayerSpec, ModelConfig
from ..ops.reference import build_cos_sin
from .latent_attention import LatentAttention
from .layout import Get, fuse_columns, pad_to, round_up, summed_linear
from .llama import _dtype_of

_ALIGN = 16  # rows between sections of the fused input projection


class FetolixLayer:
    """Weights of one layer; a looped layer is one FetolixLayer."""

    def __init__(self, spec: LayerSpec, cfg: ModelConfig, tp_rank: int, tp_world: int):
        self.mixer = LatentAttention(
            spec.mixer, cfg.hidden_size, cfg.rms_eps, tp_rank, tp_world
        )
        self.mlp = spec.mlp
        self.width = cfg.hidden_size
        self.tp_rank = tp_rank
        self.ff = self.ff_pad = 0
        if self.mlp:
            if self.mlp.width % tp_world:
                raise ValueError("TP degree must divide the feed-forward width")
            self.ff = self.mlp.width // tp_world
            self.ff_pad = round_up(self.ff, _ALIGN)
        # section -> (first row, rows) of w_in
        m = self.mixer
        self.sections: Dict[str, Tuple[int, int]] = {}
        at = 0
        for name, rows in (
            ("q", m.q_rank or m.q_dim),
            ("kv", m.spec.kv_rank + m.spec.rot_dim),
            ("gate", m.heads if m.spec.head_gate else 0),
            ("glu", 2 * self.ff_pad),
        ):
            self.sections[name] = (at, rows)
            at = round_up(at + rows, _ALIGN)
        self.in_rows = at
        self.norm: torch.Tensor = None
        self.w_in: torch.Tensor = None    # [in_rows, width]
        # output projections over column ranges of [attention | glu], summed
        self.w_out: List[torch.Tensor] = []
        self.side_gate = self.side_proj = self.side_norm = None

    def load(self, get: Get, p: str, side_dim: int) -> None:
        m = self.mixer
        self.norm = get(p + "norm1")
        sec = m.load(get, p + "mix.")
        w_in = self.norm.new_zeros(self.in_rows, self.width)
        for name in ("q", "kv", "gate"):
            at, rows = self.sections[name]
            if rows:
                w_in[at : at + rows] = sec[name]
        outs = [sec["o"]]
        if self.mlp:
            at = self.sections["glu"][0]
            mine = slice(self.tp_rank * self.ff, (self.tp_rank + 1) * self.ff)
            w_in[at : at + self.ff] = get(p + "mlp.gate")[mine]
            w_in[at + self.ff_pad : at + self.ff_pad + self.ff] = get(p + "mlp.up")[mine]
            outs.append(pad_to(get(p + "mlp.down")[:, mine], self.width, self.ff_pad))
        self.w_in = w_in
        self.w_out = fuse_columns(outs)
        if side_dim:
            self.side_gate = get(p + "side.gate")
            self.side_proj = get(p + "side.proj")
            self.side_norm = get(p + "side.norm")

    def export(self, p: str) -> Dict[str, torch.Tensor]:
        m = self.mixer
        sec = {
            n: self.w_in[at : at + rows] for n, (at, rows) in self.sections.items() if rows
        }
        w_out = torch.cat(self.w_out, 1)
        sec["o"] = w_out[:, : m.out_dim].contiguous()
        out = {p + "norm1": self.norm, **m.export(sec, p + "mix.")}
        if self.mlp:
            out[p + "mlp.gate"] = sec["glu"][: self.ff]
            out[p + "mlp.up"] = sec["glu"][self.ff_pad : self.ff_pad + self.ff]
            out[p + "mlp.down"] = w_out[:, m.out_dim : m.out_dim + self.ff]
        if self.side_gate is not None:
            out[p + "side.gate"] = self.side_gate
            out[p + "side.proj"] = self.side_proj
            out[p + "side.norm"] = self.side_norm
        return out

    def sublayers(self, h: torch.Tensor, batch: FlatBatch, cache: torch.Tensor) -> torch.Tensor:
        """attention(h) + glu(h), [N, width]."""
        m = self.mixer
        proj = ops.linear(h, self.w_in)
        mixed = torch.empty(
            h.shape[0], m.out_dim + self.ff_pad, dtype=h.dtype, device=h.device
        )

        def section(name):
            at, rows = self.sections[name]
            return proj[:, at : at + rows] if rows else None

        if self.mlp:
            ops.clamped_glu(
                section("glu"), self.mlp.limit, self.mlp.alpha, self.mlp.offset,
                mixed[:, m.out_dim :],
            )
        m.forward(
            section("q"), section("kv"), section("gate"), batch, cache,
            mixed[:, : m.out_dim],
        )
        return summed_linear(mixed, self.w_out)


class FetolixForCausalLM:
    def __init__(self, cfg: ModelConfig, ecfg: EngineConfig, device: str,
                 tp_rank: int = 0, tp_world: int = 1):
        self.cfg = cfg
        self.ecfg = ecfg
        self.device = torch.device(device)
        self.dtype = _dtype_of(cfg)
        self.tp_rank = tp_rank
        self.tp_world = tp_world
        self.layers: List[FetolixLayer] = [
            FetolixLayer(s, cfg, tp_rank, tp_world) for s in cfg.layers
        ]
        # one rotation table per distinct rotation; a speculative step may run
        # one position past the limit
        positions = min(ecfg.max_model_len, cfg.max_position) + 1
        tables: Dict[Tuple[float, int], torch.Tensor] = {}
        for layer in self.layers:
            key = (layer.mixer.spec.rope_base, layer.mixer.spec.rot_dim)
            if key not in tables:
                tables[key] = build_cos_sin(
                    positions, key[1], key[0], self.device, exact=True
                )
            layer.mixer.cos_sin = tables[key]
        self.embed: Optional[torch.Tensor] = None
        self.final_norm: Optional[torch.Tensor] = None
        self.loop_in: Optional[torch.Tensor] = None
        self.side_embed: Optional[torch.Tensor] = None
        # one latent cache per layer run, allocated by allocate_kv_cache
        self.caches: List[torch.Tensor] = []
        # TP all-reduce hook installed by the engine
        self.all_reduce = None

    # ------------------------------------------------------------- weights

    def weight_shapes(self) -> List[Tuple[str, Tuple[int, ...]]]:
        """Checkpoint tensors of the whole model."""
        cfg, w = self.cfg, self.cfg.hidden_size
        out = [("embed", (cfg.vocab_size, w)), ("final.norm", (w,))]
        if cfg.loop:
            out.append(("loop.in", (w, 2 * w)))
        if cfg.token_side_dim:
            out.append(("side.embed", (cfg.vocab_size, len(self.layers) * cfg.token_side_dim)))
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            out.append((p + "norm1", (w,)))
            out += [(p + "mix." + n, s) for n, s in layer.mixer.shapes()]
            if layer.mlp:
                ff = layer.mlp.width
                out += [(p + "mlp.gate", (ff, w)), (p + "mlp.up", (ff, w)),
                        (p + "mlp.down", (w, ff))]
            if cfg.token_side_dim:
                d = cfg.token_side_dim
                out += [(p + "side.gate", (d, w)), (p + "side.proj", (w, d)),
                        (p + "side.norm", (w,))]
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
        if self.cfg.loop:
            self.loop_in = mine("loop.in")
        if self.cfg.token_side_dim:
            self.side_embed = mine("side.embed")
        for i, layer in enumerate(self.layers):
            layer.load(mine, f"l{i}.", self.cfg.token_side_dim)

    def random_init(self, seed: int = 0) -> None:
        """Random weights of the config's shapes.  Every rank draws the same
        whole tensors and keeps its slice, so a TP group holds one model."""
        g = torch.Generator(device=self.device).manual_seed(seed)
        shapes = dict(self.weight_shapes())

        def draw(name: str) -> torch.Tensor:
            t = torch.empty(shapes[name], dtype=self.dtype, device=self.device)
            return t.fill_(1.0) if t.dim() == 1 else t.normal_(0.0, 0.02, generator=g)

        self.load_tensors(draw)

    def named_tensors(self) -> Dict[str, torch.Tensor]:
        out = {"embed": self.embed, "final.norm": self.final_norm}
        if self.loop_in is not None:
            out["loop.in"] = self.loop_in
        if self.side_embed is not None:
            out["side.embed"] = self.side_embed
        for i, layer in enumerate(self.layers):
            out.update(layer.export(f"l{i}."))
        return out

    def load_safetensors(self, path: str) -> None:
        from .weights import load_checkpoint

        load_checkpoint(self, path)

    # ------------------------------------------------------------ KV cache

    def allocate_kv_cache(self, num_blocks: int, block_size: int) -> None:
        self.caches = [
            self.layers[i].mixer.new_cache(num_blocks, block_size, self.dtype, self.device)
            for i, _ in self.cfg.layer_runs
        ]

    def kv_block_bytes(self, block_size: int) -> int:
        return sum(
            block_size * self.layers[i].mixer.row * self.dtype.itemsize
            for i, _ in self.cfg.layer_runs
        )

    # -------------------------------------------------------------- forward

    def forward(self, batch: FlatBatch, trace: Optional[list] = None) -> torch.Tensor:
        """Logits [len(batch.logit_rows), vocab] fp32; ``trace`` collects the
        residual after every layer run."""
        cfg, eps, w = self.cfg, self.cfg.rms_eps, self.cfg.hidden_size
        runs = cfg.layer_runs
        x0 = F.embedding(batch.token_ids, self.embed)
        x = x0.float()
        # what the next layer run reads: the normed residual, or, entering a
        # loop pass, the left half of [x; x0]
        entry = None
        if cfg.loop:
            entry = torch.empty(x.shape[0], 2 * w, dtype=self.dtype, device=x.device)
            entry[:, w:] = x0
        if runs and runs[0][1]:
            entry[:, :w] = x0
            h = None
        elif runs:
            h = ops.layernorm(x, self.layers[runs[0][0]].norm, eps, self.dtype)
        for r, (i, enters) in enumerate(runs):
            layer = self.layers[i]
            if enters:
                x = ops.linear(entry, self.loop_in).float()
                h = ops.layernorm(x, layer.norm, eps, self.dtype)
            y = layer.sublayers(h, batch, self.caches[r])
            if self.all_reduce is not None:
                y = self.all_reduce(y)
            nxt = runs[r + 1] if r + 1 < len(runs) else None
            if nxt is None:
                norm, out = None, None
            elif nxt[1]:
                norm, out = None, entry[:, :w]
            else:
                norm, out = self.layers[nxt[0]].norm, torch.empty_like(h)
            if cfg.token_side_dim:
                d = cfg.token_side_dim
                x, s = ops.side_gate(
                    x, y, layer.side_gate, batch.token_ids, self.side_embed, i * d
                )
                ops.residual_norm(
                    x, ops.linear(s, layer.side_proj), eps, layer.side_norm, norm, out
                )
            else:
                ops.residual_norm(x, y, eps, None, norm, out)
            h = out
            if trace is not None:
                trace.append(x.clone())
        sel = ops.layernorm(x[batch.logit_rows], self.final_norm, eps, self.dtype)
        return ops.linear(sel, self.embed).float()
