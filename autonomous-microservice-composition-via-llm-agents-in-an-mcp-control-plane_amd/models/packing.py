"""Padding of checkpoint tensors to the sizes the MFMA kernels tile by: zero rows
and columns, which leave every product exact.  Shared by the model families
whose sizes come freely from config.json."""
from __future__ import annotations

import dataclasses
from typing import Optional, Tuple

import torch

from ..ops import HEAD_SIZES, reference as ref

MAX_POS = 131072          # positions of the rotation tables when nothing else bounds them


@dataclasses.dataclass(frozen=True)
class Rotary:
    dims: int
    base: float
    scaling: Optional[Tuple[float, float, float, float]] = None   # factor, low, high, original


def up(n: int, m: int) -> int:
    return -(-n // m) * m


def head_size(d: int) -> int:
    """The head size ``d`` runs at: the next of ``HEAD_SIZES`` (larger heads,
    outside the MFMA forms, at the next multiple of 64)."""
    return next((h for h in HEAD_SIZES if h >= d), up(d, 64))


def leading(n: int, padded: int) -> torch.Tensor:
    """Row order (see ``pick_rows``) of ``n`` rows followed by zero rows."""
    at = torch.full((padded,), -1, dtype=torch.long)
    at[:n] = torch.arange(n)
    return at


def pick_rows(w: torch.Tensor, heads: int, dim: int, order: torch.Tensor) -> torch.Tensor:
    """[heads * dim, ...] -> [heads * len(order), ...] rows by ``order`` per head
    (-1: a zero row)."""
    w = w.reshape(heads, dim, *w.shape[1:])
    out = w.new_zeros(heads, len(order), *w.shape[2:])
    on = order >= 0
    out[:, on] = w[:, order[on]]
    return out.reshape(heads * len(order), *w.shape[2:])


def pad(w: torch.Tensor, *shape: int) -> torch.Tensor:
    out = w.new_zeros(*shape)
    out[tuple(slice(0, n) for n in w.shape)] = w
    return out


def rope_table(rot: Rotary, max_pos: int, pairs: int, device) -> torch.Tensor:
    """[max_pos, pairs, 2] (cos, sin); pairs that do not rotate hold (1, 0)."""
    cs = torch.zeros(max_pos, pairs, 2)
    cs[..., 0] = 1.0
    if rot.dims:
        cs[:, :rot.dims // 2] = ref.rope_cos_sin(max_pos, rot.dims, rot.base, None, rot.scaling)
    return cs.to(device)
