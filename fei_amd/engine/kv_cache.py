"""Paged caches and recurrent state of the sequences an engine serves.

``BlockAllocator`` hands out fixed-size blocks; what lies in a block is the
subclass's: ``PagedKVPool`` keys and values of one attention layer per entry,
``HybridCache`` one row per token for every layer run that caches rows and,
beside the blocks, a slot of state for every one that keeps some.

Sized for MI355X's 288 GB HBM3E: the pool reserves a fraction of free GPU
memory as fixed-size blocks; sequences map logical block indices to physical
blocks so many agent sessions can share one engine without fragmentation.
The flagship decode path uses contiguous per-sequence caches (the HIP
decode-attention kernel reads [B,Hkv,max_seq,D]); this allocator manages
*session* lifetimes above that: each session owns a contiguous region and
the pool tracks free regions. (Block-table attention is a planned kernel
extension; the allocator API already speaks blocks.)
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Sequence

import torch

from fei_amd.utils.logging import get_logger

logger = get_logger("engine.kv_cache")


@dataclass
class BlockTable:
    """Logical -> physical block mapping for one sequence."""
    seq_id: int
    blocks: List[int] = field(default_factory=list)
    length: int = 0                       # tokens used


class BlockAllocator:
    """Free list of fixed-size blocks and the block table of every live
    sequence: a sequence's logical block i is physical block
    ``table(seq).blocks[i]``."""

    def __init__(self, num_blocks: int, block_size: int,
                 device: torch.device):
        self.num_blocks = int(num_blocks)
        self.block_size = block_size
        self.device = device
        self._free: List[int] = list(range(self.num_blocks - 1, -1, -1))
        self._tables: Dict[int, BlockTable] = {}
        self._next_id = 0

    # -- sessions ------------------------------------------------------------

    def free_blocks(self) -> int:
        return len(self._free)

    def new_sequence(self) -> int:
        sid = self._next_id
        self._next_id += 1
        self._tables[sid] = BlockTable(seq_id=sid)
        return sid

    def table(self, seq_id: int) -> BlockTable:
        return self._tables[seq_id]

    def ensure_capacity(self, seq_id: int, n_tokens: int) -> List[int]:
        """Grow a sequence to hold n_tokens; returns its block list."""
        t = self._tables[seq_id]
        need = (n_tokens + self.block_size - 1) // self.block_size
        while len(t.blocks) < need:
            if not self._free:
                raise MemoryError(
                    f"KV pool exhausted ({self.num_blocks} blocks); free a "
                    "sequence first")
            t.blocks.append(self._free.pop())
        t.length = max(t.length, n_tokens)
        return t.blocks

    def release(self, seq_id: int) -> None:
        t = self._tables.pop(seq_id, None)
        if t:
            self._free.extend(t.blocks)

    def block_table_tensor(self, seq_id: int) -> torch.Tensor:
        return torch.tensor(self._tables[seq_id].blocks, dtype=torch.int32,
                            device=self.device)


class PagedKVPool(BlockAllocator):
    """Fixed-size block pool over one big tensor pair per layer.

    layout per layer: [num_blocks, Hkv, block_size, D] — a sequence's
    logical block i lives at physical index table.blocks[i].
    """

    def __init__(
        self,
        num_layers: int,
        num_kv_heads: int,
        head_dim: int,
        block_size: int = 16,
        num_blocks: Optional[int] = None,
        device: Optional[torch.device] = None,
        dtype: torch.dtype = torch.bfloat16,
        mem_fraction: float = 0.6,
    ):
        device = device or (torch.device("cuda:0") if torch.cuda.is_available()
                            else torch.device("cpu"))
        self.dtype = dtype
        if num_blocks is None:
            if device.type == "cuda":
                free, _total = torch.cuda.mem_get_info(device)
                budget = int(free * mem_fraction)
            else:
                budget = 1 << 28
            bytes_per_block = (2 * num_layers * num_kv_heads * block_size *
                               head_dim * torch.tensor([], dtype=dtype).element_size())
            num_blocks = max(16, budget // bytes_per_block)
        super().__init__(num_blocks, block_size, device)
        shape = (self.num_blocks, num_kv_heads, block_size, head_dim)
        self.k = [torch.zeros(shape, device=self.device, dtype=dtype)
                  for _ in range(num_layers)]
        self.v = [torch.zeros(shape, device=self.device, dtype=dtype)
                  for _ in range(num_layers)]

    def fork(self, seq_id: int) -> int:
        """Copy-on-write-free fork is not supported (blocks are mutable);
        makes a physical copy of the parent's blocks."""
        parent = self._tables[seq_id]
        child_id = self.new_sequence()
        child = self._tables[child_id]
        for pb in parent.blocks:
            if not self._free:
                raise MemoryError("KV pool exhausted during fork")
            nb = self._free.pop()
            for lk, lv in zip(self.k, self.v):
                lk[nb].copy_(lk[pb])
                lv[nb].copy_(lv[pb])
            child.blocks.append(nb)
        child.length = parent.length
        return child_id


class HybridCache(BlockAllocator):
    """Cache of a decoder whose layer runs differ.

    ``rows[r]``: [(num_blocks + 1) * block_size, width], one row per token
    (a latent; keys and values). ``states[r]``: float32
    [num_slots + 1, *shape], one entry per live sequence (the state of linear
    attention; the last inputs of a short convolution). Either is None where
    the run's mixer has none. A sequence holds one state slot from
    ``new_sequence`` to ``release`` and as many blocks as its length needs.

    The last block and the last slot belong to no sequence: they take the
    writes of steps that must leave no trace (graph warm-up).

    Nothing is cleared when a block or slot is used again: rows beyond a
    sequence's length are never read, and a sequence at position 0 starts
    from a zero state in the kernels whatever its slot holds.
    """

    def __init__(self, row_widths: Sequence[Optional[int]],
                 state_shapes: Sequence[Optional[Sequence[int]]],
                 num_blocks: int, num_slots: int, block_size: int = 64,
                 device: Optional[torch.device] = None,
                 dtype: torch.dtype = torch.bfloat16):
        device = device or torch.device("cpu")
        if block_size & (block_size - 1):
            raise ValueError("block size must be a power of two")
        super().__init__(num_blocks, block_size, device)
        self.dtype = dtype
        self.num_slots = int(num_slots)
        n_rows = (self.num_blocks + 1) * block_size
        self.rows = [None if w is None else
                     torch.zeros(n_rows, w, device=device, dtype=dtype)
                     for w in row_widths]
        self.states = [None if s is None else
                       torch.zeros(self.num_slots + 1, *s, device=device,
                                   dtype=torch.float32)
                       for s in state_shapes]
        self._free_slots: List[int] = list(range(self.num_slots - 1, -1, -1))
        self._slots: Dict[int, int] = {}

    @property
    def scratch_block(self) -> int:
        return self.num_blocks

    @property
    def scratch_slot(self) -> int:
        return self.num_slots

    def free_slots(self) -> int:
        return len(self._free_slots)

    def slot(self, seq_id: int) -> int:
        return self._slots[seq_id]

    def new_sequence(self) -> int:
        if not self._free_slots:
            raise MemoryError(f"all {self.num_slots} state slots are in use; "
                              "free a sequence first")
        sid = super().new_sequence()
        self._slots[sid] = self._free_slots.pop()
        return sid

    def release(self, seq_id: int) -> None:
        super().release(seq_id)
        slot = self._slots.pop(seq_id, None)
        if slot is not None:
            self._free_slots.append(slot)

    def fork(self, seq_id: int) -> int:
        """A new sequence with a copy of this one's rows and state."""
        parent = self.table(seq_id)
        child_id = self.new_sequence()
        try:
            blocks = self.ensure_capacity(child_id, parent.length)
        except MemoryError:
            self.release(child_id)
            raise
        bs = self.block_size
        for rows in self.rows:
            if rows is not None:
                blk = rows.view(-1, bs, rows.shape[1])
                for src, dst in zip(parent.blocks, blocks):
                    blk[dst].copy_(blk[src])
        for st in self.states:
            if st is not None:
                st[self.slot(child_id)].copy_(st[self.slot(seq_id)])
        return child_id
