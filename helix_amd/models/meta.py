"""What the engine hands a model with every step, and what a model tells the
engine about its cache."""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple

import numpy as np
import torch


@dataclass(frozen=True)
class KVLayer:
    """Cache geometry of one layer: pages of K [G, bs, k_dim] and of V
    [G, bs, v_dim], or [G, v_dim, bs] when v_transposed."""
    num_kv_heads: int
    k_dim: int
    v_dim: int
    v_transposed: bool = False

    def k_shape(self, block_size: int):
        return (self.num_kv_heads, block_size, self.k_dim)

    def v_shape(self, block_size: int):
        if self.v_transposed:
            return (self.num_kv_heads, self.v_dim, block_size)
        return (self.num_kv_heads, block_size, self.v_dim)


@dataclass(frozen=True)
class StateLayer:
    """Recurrent state of one layer, a fixed amount per sequence: (shape,
    dtype) of each of its tensors, dtype None = the cache's own."""
    tensors: Tuple[Tuple[Tuple[int, ...], Optional[torch.dtype]], ...]

    def bytes_per_slot(self, dtype: torch.dtype) -> int:
        return sum(int(np.prod(shape)) * torch.empty(
            0, dtype=dt or dtype).element_size() for shape, dt in self.tensors)


@dataclass
class PromptContext:
    """The cached tokens that prompt portions attend to, gathered into one
    row list. Sequence i of the group [first, last) of the batch owns the
    rows [start[i], start[i] + length[i]); its newest tokens come last.
    Starts are multiples of 8, rows between the sequences (and CONTEXT_TAIL
    after the last) repeat valid ones."""
    first: int
    last: int
    slots: torch.Tensor            # [rows] int64 cache slots
    start: torch.Tensor            # [last - first] int32
    length: torch.Tensor           # [last - first] int32


CONTEXT_TAIL = 32
CONTEXT_ROWS = 1 << 16             # rows of a group, unless one needs more


@dataclass
class PromptChunks:
    """The prompt portions cut into chunks of equal size, each portion from
    its own first token on."""
    size: int
    seq: torch.Tensor              # [n] int32 sequence of the chunk
    row: torch.Tensor              # [n] int32 its first row
    count: torch.Tensor            # [n] int32 its rows
    first: torch.Tensor            # [B + 1] int32 chunk numbers per sequence


@dataclass
class PrefillMeta:
    """Varlen prompt portions: q/k/v are the concatenated new tokens of all
    sequences. Where a sequence has earlier tokens in the cache, attention
    either gathers the full context (gather_blk/off, cu_seqlens_k carries
    the full-context boundaries) or, in models with paged_prefill, reads the
    pages itself (block_tables, seq_lens, row_seq, row_len)."""
    cu_seqlens: torch.Tensor       # [B+1] int32 (new-token boundaries)
    max_seqlen: int
    slot_mapping: torch.Tensor     # [T] int64 cache slots for new tokens
    positions: torch.Tensor        # [T] int64
    cu_seqlens_k: Optional[torch.Tensor] = None   # [B+1] int32 full context
    gather_blk: Optional[torch.Tensor] = None     # [Tk] int64
    gather_off: Optional[torch.Tensor] = None     # [Tk] int64
    block_tables: Optional[torch.Tensor] = None   # [B, max_blocks] int32
    seq_lens: Optional[torch.Tensor] = None       # [B] int32 full context
    row_seq: Optional[torch.Tensor] = None        # [T] int32 row of block_tables
    row_len: Optional[torch.Tensor] = None        # [T] int32 position + 1
    max_len: int = 0                              # host-side max(seq_lens)
    state_slots: Optional[torch.Tensor] = None    # [B] int32 recurrent state
    starts: Optional[np.ndarray] = None           # host: first new position
    ends: Optional[np.ndarray] = None             # host: seq_lens
    host_tables: Optional[np.ndarray] = None      # host: block_tables
    block_size: int = 0
    is_prefill: bool = True
    _cache: Dict = field(default_factory=dict)

    def context(self, window: int) -> List[PromptContext]:
        """Groups of sequences with what they see under a sliding window
        (0 = everything)."""
        key = ("context", window)
        if key not in self._cache:
            low = np.maximum(self.starts - window + 1, 0) if window \
                else np.zeros_like(self.starts)
            room = -(-(self.ends - low) // 8) * 8
            groups, first = [], 0
            while first < len(room):
                last = first + 1
                while last < len(room) and \
                        room[first:last + 1].sum() <= CONTEXT_ROWS:
                    last += 1
                groups.append(self._gather(first, last, low[first:last],
                                           room[first:last]))
                first = last
            self._cache[key] = groups
        return self._cache[key]

    def _gather(self, first: int, last: int, low, room) -> PromptContext:
        bs, dev = self.block_size, self.cu_seqlens.device
        length = self.ends[first:last] - low
        room = room.copy()
        start = np.concatenate([[0], np.cumsum(room)])[:-1]
        room[-1] += CONTEXT_TAIL
        which = np.repeat(np.arange(last - first), room)
        pos = low[which] + np.minimum(np.arange(len(which)) - start[which],
                                      length[which] - 1)
        slots = self.host_tables[first + which, pos // bs].astype(
            np.int64) * bs + pos % bs
        return PromptContext(first, last, _put(slots, np.int64, dev),
                             _put(start, np.int32, dev),
                             _put(length, np.int32, dev))

    def chunks(self, size: int) -> PromptChunks:
        key = ("chunks", size)
        if key not in self._cache:
            dev = self.cu_seqlens.device
            lens = self.ends - self.starts
            per = -(-lens // size)
            first = np.concatenate([[0], np.cumsum(per)])
            row0 = np.concatenate([[0], np.cumsum(lens)])
            seq = np.repeat(np.arange(len(lens)), per)
            at = (np.arange(first[-1]) - first[seq]) * size
            self._cache[key] = PromptChunks(
                size, _put(seq, np.int32, dev),
                _put(row0[seq] + at, np.int32, dev),
                _put(np.minimum(lens[seq] - at, size), np.int32, dev),
                _put(first, np.int32, dev))
        return self._cache[key]


def _put(a: np.ndarray, dtype, device) -> torch.Tensor:
    return torch.from_numpy(np.ascontiguousarray(a, dtype=dtype)).to(device)


@dataclass
class DecodeMeta:
    """One new token per running sequence."""
    block_tables: torch.Tensor     # [B, max_blocks] int32
    seq_lens: torch.Tensor         # [B] int32 (context incl. current token)
    slot_mapping: torch.Tensor     # [B] int64
    positions: torch.Tensor        # [B] int64
    max_len: int = 0               # host-side max(seq_lens) (avoids sync)
    workspace: Optional[object] = None
    state_slots: Optional[torch.Tensor] = None    # [B] int32, -1 = none
    is_prefill: bool = False


@dataclass
class MixedMeta:
    """Single decoded tokens (rows [0, num_decode)) beside prompt portions
    (the rest) in one batch."""
    decode: DecodeMeta
    prefill: PrefillMeta
    num_decode: int
    slot_mapping: torch.Tensor     # [T] int64, all rows
    positions: torch.Tensor        # [T] int64, all rows
    is_prefill: bool = True
