"""config.json of a checkpoint directory -> ModelConfig.

A reader per architecture name; the name also picks the model class
(models/__init__.py).  Every size and constant comes from the file.
"""
from __future__ import annotations

import json
import os
from typing import Callable, Dict, Optional

from ..engine.config import (
    ClampedGluSpec, LatentAttentionSpec, LayerSpec, LoopSpec, ModelConfig,
)

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


def _fetolix(d: dict) -> ModelConfig:
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


CONFIG_READERS: Dict[str, Callable[[dict], ModelConfig]] = {"Fetolix": _fetolix}


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
    return CONFIG_READERS[name](d)
