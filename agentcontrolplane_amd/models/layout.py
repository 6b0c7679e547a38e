"""Weight layout helpers: checkpoint tensors by name, and zero padding to the
sizes the kernels take."""
from __future__ import annotations

from typing import Callable

import torch

#: name -> the whole checkpoint tensor, in the model's dtype and on its device
Get = Callable[[str], torch.Tensor]


def round_up(n: int, m: int) -> int:
    return -(-n // m) * m


def pad_to(t: torch.Tensor, *shape: int) -> torch.Tensor:
    """Zero-pad each leading corner of t to shape."""
    if tuple(t.shape) == tuple(shape):
        return t
    out = t.new_zeros(shape)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


def stack_rows(sections, width: int, align: int = 16):
    """One weight from (name, [rows, width]) sections, each starting at a multiple
    of ``align`` rows; returns it and name -> (first row, rows)."""
    at, places = 0, {}
    for name, t in sections:
        places[name] = (at, t.shape[0])
        at = round_up(at + t.shape[0], align)
    out = sections[0][1].new_zeros(at, width)
    for name, t in sections:
        out[places[name][0] : places[name][0] + t.shape[0]] = t
    return out, places
