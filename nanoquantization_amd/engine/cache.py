"""What a sequence keeps between steps: blocks of a paged K/V cache and, for models with recurrent layers, one slot of
a state pool.  Both are allocated once; leasing and giving back is list bookkeeping on the host."""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import List, Optional, Sequence, Tuple

import torch


@dataclass
class Lease:
    """The cache blocks of one sequence, in token order, and its recurrent-state slot (-1: the model has none)."""
    blocks: List[int] = field(default_factory=list)
    slot: int = -1


class PagedKVCache:
    """Blocks of `block_size` tokens, [blocks, kv_heads, block_size, head_dim] per layer for K and V.  Uniform models
    hold all layers in one tensor ([layers, ...]); with `layer_shapes` -- (kv_heads, key row, value row) per layer run,
    None for a run without attention, a value row of 0 where keys and values share their row -- every run has tensors of its own size, all of them indexed by the same block
    numbers.  Rows may be wider than a head (padding stays zero: the writers never touch it)."""

    def __init__(self, num_layers: int, num_blocks: int, block_size: int, num_kv_heads: int = 0, head_dim: int = 0,
                 dtype: torch.dtype = torch.bfloat16, device: "torch.device | str" = "cuda",
                 layer_shapes: Optional[Sequence[Optional[Tuple[int, int, int]]]] = None):
        self.block_size = block_size
        self.num_blocks = num_blocks
        if layer_shapes is None:
            shape = (num_layers, num_blocks, num_kv_heads, block_size, head_dim)
            self.k = torch.zeros(shape, dtype=dtype, device=device)
            self.v = torch.zeros(shape, dtype=dtype, device=device)
        else:
            assert len(layer_shapes) == num_layers
            mk = lambda s, w: None if s is None else torch.zeros(num_blocks, s[0], block_size, s[w], dtype=dtype, device=device)
            self.k = [mk(s, 1) for s in layer_shapes]
            self.v = [mk(s, 2) for s in layer_shapes]
        self.free: List[int] = list(range(num_blocks - 1, -1, -1))

    def allocate(self, n: int) -> List[int]:
        if n > len(self.free):
            raise RuntimeError(f"KV cache exhausted: {n} blocks wanted, {len(self.free)} free")
        return [self.free.pop() for _ in range(n)]

    def release(self, blocks: List[int]) -> None:
        self.free.extend(reversed(blocks))


class RecurrentStateCache:
    """Recurrent state of `num_slots` sequences: fp32 [slots, *shape] per layer run (`run_shapes`, None for a run without
    state), and for runs behind a short convolution the last inputs of that, `tail` [slots, *tail shape].  A slot is never cleared: the kernels take the state before position 0 as zero
    whatever the slot holds, so handing a slot on costs nothing and leaks nothing."""

    def __init__(self, num_slots: int, run_shapes: Sequence[Optional[Tuple[int, ...]]], device: "torch.device | str",
                 tail_shapes: Optional[Sequence[Optional[Tuple[int, ...]]]] = None):
        self.num_slots = num_slots
        pool = lambda s: None if s is None else torch.zeros(num_slots, *s, dtype=torch.float32, device=device)
        self.state = [pool(s) for s in run_shapes]
        self.tail = [pool(s) for s in tail_shapes or [None] * len(self.state)]
        self.free: List[int] = list(range(num_slots - 1, -1, -1))

    def allocate(self) -> int:
        if not self.free:
            raise RuntimeError(f"all {self.num_slots} recurrent-state slots are in use")
        return self.free.pop()

    def release(self, slot: int) -> None:
        self.free.append(slot)
