"""Weight layout helpers: checkpoint tensors by name, and zero padding to the
sizes the kernels take."""
from __future__ import annotations

from typing import Callable, List, Optional

import torch

from .. import ops

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


def section_bias(w: torch.Tensor, places, biases) -> torch.Tensor:
    """Bias over the rows of a stack_rows() weight, zero in sections without one."""
    out = w.new_zeros(w.shape[0])
    for name, b in biases.items():
        at = places[name][0]
        out[at : at + b.shape[0]] = b
    return out


def pair_halves(t: torch.Tensor, dims: int, axis: int = -1) -> torch.Tensor:
    """Reorder the first ``dims`` entries of an axis from [u.. | v..] to (u, v) pairs: a
    rotation of i with i + dims/2 becomes one of 2i with 2i + 1.  Scores do not change
    if query and key dimensions move alike."""
    at = torch.arange(t.shape[axis], device=t.device)
    at[:dims] = at[:dims].view(2, -1).t().flatten()
    return t.index_select(axis, at)


def unpair_halves(t: torch.Tensor, dims: int, axis: int = -1) -> torch.Tensor:
    """Inverse of pair_halves()."""
    at = torch.arange(t.shape[axis], device=t.device)
    at[:dims] = at[:dims].view(-1, 2).t().flatten()
    return t.index_select(axis, at)


#: the longest inner dimension of a fused output projection: beyond it the library's
#: small-batch kernels slow down more than a second GEMM costs
_FUSED_OUT = 16384


def fuse_columns(blocks: List[torch.Tensor]) -> List[torch.Tensor]:
    """Weights [width, k] whose products are summed: one weight if it is not too long."""
    if sum(b.shape[1] for b in blocks) <= _FUSED_OUT:
        blocks = [torch.cat(blocks, 1)]
    return [b.contiguous() for b in blocks]


def summed_linear(x: torch.Tensor, blocks: List[torch.Tensor],
                  bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """x [N, sum of k] times the blocks of fuse_columns()."""
    at = blocks[0].shape[1]
    y = ops.linear(x[:, :at], blocks[0], bias)
    for b in blocks[1:]:
        ops.linear_add_(y, x[:, at : at + b.shape[1]], b)
        at += b.shape[1]
    return y
