"""Paged KV cache resident in HBM + block allocator with prefix sharing.

Layout (one allocation): ``[layers, 2(K|V), num_blocks, kv_heads/tp, 64, head_dim]``
bf16.  A block holds one 64-key attention tile of one kv head contiguously
(16 KiB at head_dim 128), which is exactly what ``csrc/attention.hip`` stages
with 16 LDS-DMA wave-instructions.  Sized from free HBM (288 GB per MI355X):
Llama-3-8B needs 128 KiB per token, so ~200 GB holds ~1.6 M tokens.

Blocks are reference counted so many requests can share the registry-prompt
prefix blocks (prefix caching).

A model whose cached layers differ in head count or head size, whose keys and
values differ, or that runs a layer more than once (each run caches its own keys)
gives one (kv_heads, key_dim, value_dim) per cached layer instead
(``KVCache.from_specs``): same blocks and block ids, one stacked tensor per
distinct (kv_heads, dim).  Latent attention caches one row per token that holds
both (value_dim 0).
"""
from __future__ import annotations

from typing import List, Optional

import torch

from .. import ops
from . import native
from .batch import BLOCK_SIZE

if native.available():
    OutOfBlocks = native.OutOfBlocks
else:
    class OutOfBlocks(RuntimeError):
        pass


class BlockAllocator:
    """Free-list allocator with refcounts.  The engine uses the C++ one
    (``native.NativeBlockAllocator``, csrc/runtime/runtime.cpp) when built;
    this is the reference implementation and CPU fallback."""

    def __init__(self, num_blocks: int):
        self.num_blocks = num_blocks
        self._free: List[int] = list(range(num_blocks - 1, -1, -1))
        self._ref = [0] * num_blocks

    @property
    def num_free(self) -> int:
        return len(self._free)

    def alloc(self, n: int) -> List[int]:
        if n > len(self._free):
            raise OutOfBlocks(f"need {n} KV blocks, {len(self._free)} free")
        out = [self._free.pop() for _ in range(n)]
        for b in out:
            self._ref[b] = 1
        return out

    def incref(self, blocks: List[int]):
        for b in blocks:
            if self._ref[b] <= 0:
                raise RuntimeError(f"incref of free block {b}")
            self._ref[b] += 1

    def free(self, blocks: List[int]):
        for b in blocks:
            if self._ref[b] <= 0:
                raise RuntimeError(f"double free of block {b}")
            self._ref[b] -= 1
            if self._ref[b] == 0:
                self._free.append(b)

    def refcount(self, b: int) -> int:
        return self._ref[b]

    def utilization(self) -> float:
        return 1.0 - len(self._free) / max(1, self.num_blocks)


def make_allocator(num_blocks: int):
    if native.available():
        return native.NativeBlockAllocator(num_blocks)
    return BlockAllocator(num_blocks)


class KVCache:
    def __init__(self, layers: int, kv_heads: int, head_dim: int, num_blocks: int, device,
                 dtype=torch.bfloat16):
        self.layers, self.kv_heads, self.head_dim = layers, kv_heads, head_dim
        self.num_blocks = num_blocks
        self.data = torch.zeros(layers, 2, num_blocks, kv_heads, BLOCK_SIZE, head_dim,
                                device=device, dtype=dtype)
        self.stacks = [self.data]              # every tensor of the cache, [n, c, num_blocks, ...]
        self._layer = [(self.data[l, 0], self.data[l, 1]) for l in range(layers)]
        self.allocator = make_allocator(num_blocks)

    @classmethod
    def from_specs(cls, specs, num_blocks: int, device, dtype=torch.bfloat16) -> "KVCache":
        """``specs``: (kv_heads, key_dim, value_dim) of every cached layer; value_dim
        0: the values are part of the keys, the layer has no value tensor."""
        self = cls.__new__(cls)
        self.layers, self.num_blocks, self.data = len(specs), num_blocks, None
        place, count = [], {}
        for h, dk, dv in specs:
            for d in (dk, dv):
                if d == 0:
                    place.append(None)
                    continue
                place.append(((h, d), count.get((h, d), 0)))
                count[(h, d)] = count.get((h, d), 0) + 1
        stack = {(h, d): torch.zeros(n, 1, num_blocks, h, BLOCK_SIZE, d, device=device, dtype=dtype)
                 for (h, d), n in count.items()}
        self.stacks = list(stack.values())
        at = [None if p is None else stack[p[0]][p[1], 0] for p in place]
        self._layer = list(zip(at[0::2], at[1::2]))
        self.allocator = make_allocator(num_blocks)
        return self

    @classmethod
    def for_model(cls, model, num_blocks: Optional[int] = None, budget_bytes: Optional[int] = None):
        """The cache of ``model``: its ``kv_specs`` when it has them, else equal
        layers from its config.  ``num_blocks`` None: sized from free memory."""
        specs = getattr(model, "kv_specs", None)
        if specs is None:
            cfg = model.cfg
            if num_blocks is not None:
                return cls(cfg.layers, model.hkv, cfg.head_dim, num_blocks, model.device)
            return cls.sized_for(cfg.layers, model.hkv, cfg.head_dim, model.device,
                                 budget_bytes=budget_bytes)
        if num_blocks is None:
            size = torch.empty(0, dtype=model.dtype).element_size()
            per = sum(h * (dk + dv) for h, dk, dv in specs) * BLOCK_SIZE * size
            num_blocks = cls._blocks_in_budget(per, model.device, budget_bytes)
        return cls.from_specs(specs, num_blocks, model.device, model.dtype)

    def layer(self, l: int):
        return self._layer[l]

    def copy_blocks(self, src, dst) -> None:
        """Block src[i] -> dst[i] in every cached layer (negative pairs: none)."""
        for t in self.stacks:
            ops.copy_blocks(t, src, dst)

    @property
    def nbytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.stacks)

    @staticmethod
    def bytes_per_block(layers, kv_heads, head_dim, dtype_bytes=2) -> int:
        return layers * 2 * kv_heads * BLOCK_SIZE * head_dim * dtype_bytes

    @classmethod
    def sized_for(cls, layers, kv_heads, head_dim, device, budget_bytes: Optional[int] = None,
                  max_blocks: Optional[int] = None, reserve_frac: float = 0.1):
        per = cls.bytes_per_block(layers, kv_heads, head_dim)
        n = cls._blocks_in_budget(per, device, budget_bytes, reserve_frac)
        if max_blocks is not None:
            n = min(n, max_blocks)
        return cls(layers, kv_heads, head_dim, n, device)

    @staticmethod
    def _blocks_in_budget(per: int, device, budget_bytes: Optional[int],
                          reserve_frac: float = 0.1) -> int:
        dev = torch.device(device)
        if budget_bytes is None:
            if dev.type == "cuda":
                free, total = torch.cuda.mem_get_info(dev)
                budget_bytes = int(free - reserve_frac * total)
            else:
                budget_bytes = 256 * per
        return int(max(16, budget_bytes // per))
