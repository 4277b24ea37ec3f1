"""One step of many sequences: the batch a model runs, and its runner.

A step takes, for each of several sequences, the next tokens of that
sequence: one token of a sequence that decodes, a portion of any length of
one that still reads its prompt. ``RaggedBatch`` packs them into flat rows,
decoding sequences first, so that every row-wise operation (projections,
norms, feed-forwards) runs once over all rows, and each mixer runs its decode
kernels over the first ``n_dec`` rows and its prompt kernels over the rest.

``StepRunner`` owns the cache and the bookkeeping of positions. Everything
that runs such a model goes through it: LocalEngine, the session scheduler
and the trace runner.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Sequence, Tuple

import numpy as np
import torch

from fei_amd.engine.kv_cache import HybridCache

CHUNK = 64           # tokens per chunk of the linear-attention prompt kernels
Q_TILE = 128         # query rows per workgroup of the prompt attention kernel


@dataclass
class RaggedBatch:
    """Device tensors of one step. Sequences are numbered 0 .. n_seq-1 in row
    order, the ``n_dec`` single-token ones first."""
    tokens: torch.Tensor               # [T] int64
    pos: torch.Tensor                  # [T] int32
    row_seq: torch.Tensor              # [T] int32, sequence of a row
    table: torch.Tensor                # [n_seq, W] int32, physical blocks
    slots: torch.Tensor                # [n_seq] int32
    n_dec: int
    # prompt portions, host side: (first row, rows, first position)
    portions: List[Tuple[int, int, int]] = field(default_factory=list)
    want_rows: Optional[torch.Tensor] = None     # [n] int64; None = all rows
    # device tensors that depend on the portions, by key (see below)
    _plans: Dict[object, object] = field(default_factory=dict)

    @property
    def n_rows(self) -> int:
        return self.tokens.shape[0]

    def _upload(self, rows, width: int) -> torch.Tensor:
        t = torch.from_numpy(np.asarray(rows, dtype=np.int32))
        return t.view(-1, width).to(self.tokens.device)

    def span_plan(self):
        """The prompt portions [first row, rows, first position], and their
        query tiles [portion, first row in it]."""
        if "spans" not in self._plans:
            tiles = [[p, q] for p, (_, n, _) in enumerate(self.portions)
                     for q in range(0, n, Q_TILE)]
            self._plans["spans"] = (self._upload(self.portions, 3),
                                    self._upload(tiles, 2))
        return self._plans["spans"]

    def key_plan(self, window: Optional[int]):
        """What the prompt portions read through a window: per portion
        [first row, rows, first position, first key position, first packed
        key], the number of packed keys, the query tiles [portion, first row
        in it], and the portion of every packed key."""
        key = ("keys", window)
        if key not in self._plans:
            spans, tiles, owner, at = [], [], [], 0
            for p, (row, n, pos0) in enumerate(self.portions):
                k0 = 0 if window is None else max(0, pos0 - window + 1)
                spans.append([row, n, pos0, k0, at])
                n_keys = pos0 + n - k0
                owner.append(np.full(n_keys, p, dtype=np.int32))
                at += n_keys
                tiles += [[p, q] for q in range(0, n, Q_TILE)]
            self._plans[key] = (self._upload(spans, 5), at,
                                self._upload(tiles, 2),
                                self._upload(np.concatenate(owner), 1).view(-1))
        return self._plans[key]

    def chunk_plan(self):
        """Chunks of the prompt portions [portion, first row, rows], and per
        portion [first chunk, chunks, first position, state slot index]."""
        if "chunks" not in self._plans:
            chunks, spans = [], []
            for p, (row, n, pos0) in enumerate(self.portions):
                first = len(chunks)
                chunks += [[p, row + c, min(CHUNK, n - c)]
                           for c in range(0, n, CHUNK)]
                spans.append([first, len(chunks) - first, pos0,
                              self.n_dec + p])
            self._plans["chunks"] = (self._upload(chunks, 3),
                                     self._upload(spans, 4))
        return self._plans["chunks"]


@dataclass
class StepEntry:
    seq: int                           # sequence id of the runner's cache
    tokens: Sequence[int]
    want: Sequence[int] = ()           # places in tokens whose logits to give


class StepRunner:
    def __init__(self, model, num_blocks: int, num_slots: int,
                 block_size: int = 64):
        self.model = model
        self.device = model.device
        self.cache: HybridCache = model.new_cache(num_blocks, num_slots,
                                                  block_size)
        self.length: Dict[int, int] = {}      # tokens run, by sequence

    # -- sequences -----------------------------------------------------------

    def admit(self, reserve: int = 0) -> int:
        """A new sequence with blocks for ``reserve`` tokens; MemoryError if
        slots or blocks are short (nothing is kept then)."""
        sid = self.cache.new_sequence()
        try:
            self.cache.ensure_capacity(sid, reserve)
        except MemoryError:
            self.cache.release(sid)
            raise
        self.length[sid] = 0
        return sid

    def release(self, sid: int) -> None:
        self.cache.release(sid)
        self.length.pop(sid, None)

    def set_length(self, sid: int, n: int) -> None:
        """The sequence's next token is at position ``n``: 0 to start over,
        or what the caller ran on the device by itself."""
        self.length[sid] = n

    # -- steps ---------------------------------------------------------------

    def _tables(self, seqs: Sequence[int]) -> Tuple[torch.Tensor, torch.Tensor]:
        blocks = [self.cache.table(s).blocks for s in seqs]
        W = max(max((len(b) for b in blocks), default=1), 1)
        host = np.full((len(seqs), W), self.cache.scratch_block, np.int32)
        for i, b in enumerate(blocks):
            host[i, :len(b)] = b
        table = torch.from_numpy(host)
        slots = torch.tensor([self.cache.slot(s) for s in seqs],
                             dtype=torch.int32)
        return table.to(self.device), slots.to(self.device)

    def build(self, entries: Sequence[StepEntry],
              all_rows: bool = False) -> RaggedBatch:
        """Reserve cache room for the entries and pack them. Wanted rows are
        in the order of the entries (all rows in packed order if
        ``all_rows``)."""
        if not entries:
            raise ValueError("a step needs at least one entry")
        seqs = [e.seq for e in entries]
        if len(set(seqs)) != len(seqs):
            raise ValueError("a sequence may appear once in a step")
        V = self.model.spec.vocab_size
        limit = self.model.max_seq_len
        for e in entries:
            if not len(e.tokens):
                raise ValueError("an entry needs at least one token")
            t = np.asarray(e.tokens)
            if t.min() < 0 or t.max() >= V:
                raise ValueError(f"token outside the vocabulary of {V}")
            if any(w < 0 or w >= len(e.tokens) for w in e.want):
                raise ValueError("a wanted place is outside the entry")
            if self.length[e.seq] + len(e.tokens) > limit:
                raise ValueError(f"sequence longer than {limit} tokens")
        for e in entries:
            self.cache.ensure_capacity(e.seq,
                                       self.length[e.seq] + len(e.tokens))
        order = sorted(range(len(entries)),
                       key=lambda i: len(entries[i].tokens) > 1)
        # token, position and sequence of every row
        meta = np.empty((3, sum(len(e.tokens) for e in entries)), np.int32)
        portions: List[Tuple[int, int, int]] = []
        first_row: Dict[int, int] = {}
        n_dec = row = 0
        for s, i in enumerate(order):
            e = entries[i]
            p0, n = self.length[e.seq], len(e.tokens)
            first_row[i] = row
            if n == 1:
                n_dec += 1
            else:
                portions.append((row, n, p0))
            meta[0, row:row + n] = e.tokens
            meta[1, row:row + n] = np.arange(p0, p0 + n)
            meta[2, row:row + n] = s
            row += n
        table, slots = self._tables([entries[i].seq for i in order])
        want = [first_row[i] + w for i, e in enumerate(entries)
                for w in e.want]
        rows = torch.from_numpy(meta).to(self.device)
        return RaggedBatch(
            tokens=rows[0].long(), pos=rows[1], row_seq=rows[2], table=table,
            slots=slots, n_dec=n_dec, portions=portions,
            want_rows=None if all_rows else torch.tensor(
                want, dtype=torch.int64, device=self.device))

    @torch.no_grad()
    def step(self, entries: Sequence[StepEntry],
             all_rows: bool = False) -> torch.Tensor:
        """Run one batch; float32 logits [wanted, vocab]."""
        batch = self.build(entries, all_rows)
        logits = self.model.forward(batch, self.cache)
        for e in entries:
            self.length[e.seq] += len(e.tokens)
        return logits

    def decode_batch(self, seqs: Sequence[int], room: int,
                     tokens: Optional[Sequence[int]] = None) -> RaggedBatch:
        """A batch of one token per sequence whose ``tokens`` and ``pos`` the
        caller advances in place; blocks for ``room`` more tokens are
        reserved. The caller reports what it ran with ``set_length``."""
        for s in seqs:
            if self.length[s] + room > self.model.max_seq_len:
                raise ValueError("sequence longer than "
                                 f"{self.model.max_seq_len} tokens")
            self.cache.ensure_capacity(s, self.length[s] + room)
        table, slots = self._tables(seqs)
        dev = self.device
        return RaggedBatch(
            tokens=torch.tensor(list(tokens) if tokens is not None
                                else [0] * len(seqs),
                                dtype=torch.int64, device=dev),
            pos=torch.tensor([self.length[s] for s in seqs],
                             dtype=torch.int32, device=dev),
            row_seq=torch.arange(len(seqs), dtype=torch.int32, device=dev),
            table=table, slots=slots, n_dec=len(seqs))
