"""config.json of a checkpoint directory -> ModelConfig.

A reader per architecture name; the name also picks the model class
(models/__init__.py).  Every size and constant comes from the file.
"""
from __future__ import annotations

import dataclasses
import json
import os
from typing import Callable, Dict, Optional, Tuple

from ..engine.config import (
    ClampedGluSpec, DistanceBias, ExpertsSpec, GatedDeltaSpec, GroupedAttentionSpec,
    LatentAttentionSpec, LayerSpec, LoopSpec, ModelConfig, QueryTemperature, RotarySpec,
    WavelengthScaling, YarnScaling, gelu_glu, silu_glu,
)
from .weights import tensor_shape

#: a tensor's shape in the checkpoint, by name: for sizes only the weights have
Shape = Callable[[str], Tuple[int, ...]]

#: the rotation tables bound positions; the design itself sets no limit, so
#: the engine's max_model_len decides
_UNBOUNDED = 1 << 20


def _latent_attention(m: dict, *, low_rank_query: bool, window: bool) -> LatentAttentionSpec:
    if m["rot"]["dims"] != m["rot_dim"]:
        raise ValueError("latent attention rotates all of its rot_dim dimensions")
    return LatentAttentionSpec(
        heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"], vdim=m["vdim"],
        kv_rank=m["kv_rank"], scale=m["scale"], rope_base=m["rot"]["base"],
        q_rank=m["q_rank"] if low_rank_query else None,
        window=m["mask"]["size"] if window else None,
    )


#: Fetolix mixer type -> spec reader
_FETOLIX_MIXERS = {
    "latent_attention": lambda m: _latent_attention(m, low_rank_query=True, window=True),
    "latent_attention_2": lambda m: _latent_attention(m, low_rank_query=False, window=False),
}


def _fetolix_mlp(mlp: Optional[dict]) -> Optional[ClampedGluSpec]:
    if mlp is None:
        return None
    if mlp["kind"] != "dense":
        raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
    return ClampedGluSpec(width=mlp["ff"], limit=mlp["limit"])


def _fetolix(d: dict, shape: Shape) -> ModelConfig:
    layers = []
    for entry in d["layers"]:
        if entry["type"] not in _FETOLIX_MIXERS:
            raise ValueError(f"unknown mixer type {entry['type']!r}")
        layers.append(LayerSpec(
            mixer=_FETOLIX_MIXERS[entry["type"]](entry["mixer"]),
            mlp=_fetolix_mlp(entry.get("mlp")),
        ))
    loop = d.get("loop")
    first = layers[0].mixer
    return ModelConfig(
        name="Fetolix", architecture="Fetolix", vocab_size=d["vocab"],
        hidden_size=d["width"], num_layers=len(layers), num_heads=first.heads,
        num_kv_heads=1, head_dim=first.dim + first.rot_dim,
        intermediate_size=max((x.mlp.width for x in layers if x.mlp), default=0),
        rms_eps=d["norm"]["eps"], max_position=_UNBOUNDED, tie_embeddings=True,
        layers=tuple(layers),
        loop=LoopSpec(loop["start"], loop["stop"], loop["times"]) if loop else None,
        token_side_dim=(d.get("token_side") or {}).get("dim", 0),
    )


def _channel_delta(m: dict, shape: Shape, p: str) -> GatedDeltaSpec:
    return GatedDeltaSpec(
        heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"],
        conv=m["conv"], decay_rank=shape(p + "a1")[0], gate_rank=shape(p + "g1")[0],
    )


def _head_delta(m: dict) -> GatedDeltaSpec:
    return GatedDeltaSpec(
        heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"],
        conv=m["conv"], head_decay=True, gate_silu=True,
    )


def _grouped_attention(m: dict, shape: Shape, p: str) -> GroupedAttentionSpec:
    return GroupedAttentionSpec(
        heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"],
        scale=m["scale"], softcap=m["softcap"], window=m["mask"]["size"],
        keep_first=m["mask"]["keep_first"], kv_from=m.get("kv_from"),
    )


#: Tezinex mixer type -> spec reader
_TEZINEX_MIXERS = {"channel_delta": _channel_delta, "attention": _grouped_attention}


def _tezinex_mlp(mlp: Optional[dict]) -> Optional[ClampedGluSpec]:
    if mlp is None:
        return None
    if mlp["kind"] != "dense":
        raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
    return silu_glu(mlp["ff"])


def _check_borrowed_keys(layers) -> None:
    for i, layer in enumerate(layers):
        j = getattr(layer.mixer, "kv_from", None)
        if j is None:
            continue
        m, owner = layer.mixer, layers[j].mixer if 0 <= j < i else None
        if not isinstance(owner, GroupedAttentionSpec) or owner.kv_from is not None:
            raise ValueError(f"layer {i}: layer {j} has no keys and values to use")
        if (m.kv_heads, m.dim, m.vdim) != (owner.kv_heads, owner.dim, owner.vdim):
            raise ValueError(f"layer {i}: its key/value heads differ from layer {j}'s")


def _tezinex(d: dict, shape: Shape) -> ModelConfig:
    layers = []
    for i, entry in enumerate(d["layers"]):
        if entry["type"] not in _TEZINEX_MIXERS:
            raise ValueError(f"unknown mixer type {entry['type']!r}")
        m = _TEZINEX_MIXERS[entry["type"]](entry["mixer"], shape, f"l{i}.mix.")
        if m.heads % m.kv_heads:
            raise ValueError(f"layer {i}: kv_heads must divide heads")
        layers.append(LayerSpec(mixer=m, mlp=_tezinex_mlp(entry.get("mlp")), sandwich=True))
    _check_borrowed_keys(layers)
    first = layers[0].mixer
    return ModelConfig(
        name="Tezinex", architecture="Tezinex", vocab_size=d["vocab"],
        hidden_size=d["width"], num_layers=len(layers), num_heads=first.heads,
        num_kv_heads=first.kv_heads, head_dim=first.dim,
        intermediate_size=max((x.mlp.width for x in layers if x.mlp), default=0),
        rms_eps=d["norm"]["eps"], max_position=_UNBOUNDED, tie_embeddings=True,
        layers=tuple(layers), residual_mult=d["residual_mult"], depth_average=True,
        position_base=10000.0, logit_softcap=d["logit_softcap"],
    )


def _biased_attention(m: dict, shape: Shape, p: str) -> GroupedAttentionSpec:
    reach, buckets = m["bias_max"], shape(p + "rel")[0]
    if buckets < 2 or reach <= buckets // 2:
        raise ValueError("distance buckets must reach beyond their first half")
    return GroupedAttentionSpec(
        heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"],
        scale=m["scale"], bias=True, out_bias=True, sink=False, sigmoid=True, conv=m["conv"],
        qk_norm=True, v_norm=True, distance_bias=DistanceBias(buckets, reach),
        q_temp=QueryTemperature(m["q_temp"]["coef"], m["q_temp"]["every"]),
    )


def _yarn_latent_attention(m: dict, shape: Shape, p: str) -> LatentAttentionSpec:
    rot, s = m["rot"], m["rot"]["scaling"]
    if rot["dims"] != m["rot_dim"]:
        raise ValueError("latent attention rotates all of its rot_dim dimensions")
    return LatentAttentionSpec(
        heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"], vdim=m["vdim"],
        kv_rank=m["kv_rank"], scale=m["scale"], rope_base=rot["base"], rope_half=True,
        rope_scaling=YarnScaling(s["factor"], s["original"], s["fast"], s["slow"]),
        window=m["mask"]["size"], head_gate=False, sink=True,
    )


def _rotated_attention(m: dict, shape: Shape, p: str) -> GroupedAttentionSpec:
    rot, s = m["rot"], m["rot"]["scaling"]
    if rot["dims"] % 2 or rot["dims"] > m["dim"]:
        raise ValueError("rot.dims must be even and at most dim")
    return GroupedAttentionSpec(
        heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"],
        scale=m["scale"], softcap=m["softcap"], window=m["mask"]["size"], bias=False,
        sink=False, head_temp=True, head_gate=True, rotary=RotarySpec(
            rot["base"], rot["dims"],
            WavelengthScaling(s["factor"], s["low"], s["high"], s["original"]),
        ),
    )


#: Lobuvik mixer type -> spec reader
_LOBUVIK_MIXERS = {
    "attention": _biased_attention,
    "latent_attention": _yarn_latent_attention,
    "attention_2": _rotated_attention,
}


def _lobuvik_mlp(mlp: Optional[dict]):
    if mlp is None:
        return None
    if mlp["kind"] == "dense":
        return gelu_glu(mlp["ff"])
    if mlp["kind"] != "moe":
        raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")

    def glu(d: dict) -> ClampedGluSpec:
        return ClampedGluSpec(width=d["ff"], limit=d["limit"])

    router, shared = mlp["router"], mlp.get("shared")
    if not 0 < router["top"] <= router["experts"]:
        raise ValueError("a token uses between 1 and all experts")
    return ExpertsSpec(
        experts=router["experts"], top=router["top"], expert=glu(mlp["expert"]),
        shared=glu(shared) if shared else None,
    )


def _lobuvik(d: dict, shape: Shape) -> ModelConfig:
    layers = []
    for i, entry in enumerate(d["layers"]):
        if entry["type"] not in _LOBUVIK_MIXERS:
            raise ValueError(f"unknown mixer type {entry['type']!r}")
        m = _LOBUVIK_MIXERS[entry["type"]](entry["mixer"], shape, f"l{i}.mix.")
        if isinstance(m, GroupedAttentionSpec) and m.heads % m.kv_heads:
            raise ValueError(f"layer {i}: kv_heads must divide heads")
        layers.append(LayerSpec(mixer=m, mlp=_lobuvik_mlp(entry.get("mlp")), mlp_norm=True))
    first = layers[0].mixer
    return ModelConfig(
        name="Lobuvik", architecture="Lobuvik", vocab_size=d["vocab"],
        hidden_size=d["width"], num_layers=len(layers), num_heads=first.heads,
        num_kv_heads=getattr(first, "kv_heads", 1), head_dim=first.dim,
        intermediate_size=max((x.mlp.width for x in layers if x.mlp), default=0),
        rms_eps=d["norm"]["eps"], max_position=_UNBOUNDED, layers=tuple(layers),
        embed_scale=d["embedding"]["scale"],
    )


def _talking_attention(m: dict) -> GroupedAttentionSpec:
    rot, s = m["rot"], m["rot"]["scaling"]
    if rot["dims"] % 2 or rot["dims"] > m["dim"]:
        raise ValueError("rot.dims must be even and at most dim")
    return GroupedAttentionSpec(
        heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"],
        scale=m["scale"], chunk=m["mask"]["size"], bias=False, sink=False, row_norm=True,
        talk=True, rotary=RotarySpec(
            rot["base"], rot["dims"],
            YarnScaling(s["factor"], s["original"], s["fast"], s["slow"]),
        ),
    )


#: Noganex mixer type -> spec reader
_NOGANEX_MIXERS = {"attention": _talking_attention, "delta": _head_delta}


def _noganex_mlp(mlp: Optional[dict]):
    if mlp is None:
        return None
    if mlp["kind"] == "dense":
        return gelu_glu(mlp["ff"], bias=True)
    if mlp["kind"] != "moe":
        raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
    router, shared = mlp["router"], mlp.get("shared")
    if not 0 < router["top"] <= router["experts"]:
        raise ValueError("a token uses between 1 and all experts")
    return ExpertsSpec(
        experts=router["experts"], top=router["top"], expert=silu_glu(mlp["expert"]["ff"]),
        shared=silu_glu(shared["ff"]) if shared else None, router_bias=False, sigmoid=True,
        correction=True, scale=router["scale"],
    )


def _check_shared_weights(layers) -> None:
    for i, layer in enumerate(layers):
        j = layer.weights_of
        if j is None:
            continue
        owner = layers[j] if 0 <= j < len(layers) else None
        if owner is None or owner.weights_of is not None:
            raise ValueError(f"layer {i}: layer {j} has no weights to use")
        if dataclasses.replace(layer, weights_of=None) != owner:
            raise ValueError(f"layer {i} differs from layer {j}, whose weights it uses")


def _noganex(d: dict, shape: Shape) -> ModelConfig:
    layers = []
    for i, entry in enumerate(d["layers"]):
        if entry["type"] not in _NOGANEX_MIXERS:
            raise ValueError(f"unknown mixer type {entry['type']!r}")
        m = _NOGANEX_MIXERS[entry["type"]](entry["mixer"])
        if m.heads % m.kv_heads:
            raise ValueError(f"layer {i}: kv_heads must divide heads")
        layers.append(LayerSpec(
            mixer=m, mlp=_noganex_mlp(entry.get("mlp")), norm_out=True, gated=True,
            weights_of=entry.get("weights_of"),
        ))
    _check_shared_weights(layers)
    first = layers[0].mixer
    return ModelConfig(
        name="Noganex", architecture="Noganex", vocab_size=d["vocab"],
        hidden_size=d["width"], num_layers=len(layers), num_heads=first.heads,
        num_kv_heads=first.kv_heads, head_dim=first.dim,
        intermediate_size=max((x.mlp.width for x in layers if x.mlp), default=0),
        rms_eps=d["norm"]["eps"], max_position=_UNBOUNDED, layers=tuple(layers),
        logit_scale=d["logit_scale"],
    )


CONFIG_READERS: Dict[str, Callable[[dict, Shape], ModelConfig]] = {
    "Fetolix": _fetolix,
    "Tezinex": _tezinex,
    "Lobuvik": _lobuvik,
    "Noganex": _noganex,
}


def read_architecture(path: str) -> Optional[str]:
    """The registered architecture a checkpoint directory names, or None."""
    try:
        with open(os.path.join(path, "config.json")) as f:
            name = json.load(f).get("architecture")
    except (OSError, ValueError, AttributeError):
        return None
    return name if name in CONFIG_READERS else None


def read_model_config(path: str) -> ModelConfig:
    with open(os.path.join(path, "config.json")) as f:
        d = json.load(f)
    name = d.get("architecture")
    if name not in CONFIG_READERS:
        raise ValueError(
            f"{path}/config.json names architecture {name!r}; have {sorted(CONFIG_READERS)}"
        )
    return CONFIG_READERS[name](d, lambda tensor: tensor_shape(path, tensor))
