"""What the engine hands a model with every step, and what a model tells the
engine about its cache."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

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
    is_prefill: bool = True


@dataclass
class DecodeMeta:
    """One new token per running sequence."""
    block_tables: torch.Tensor     # [B, max_blocks] int32
    seq_lens: torch.Tensor         # [B] int32 (context incl. current token)
    slot_mapping: torch.Tensor     # [B] int64
    positions: torch.Tensor        # [B] int64
    max_len: int = 0               # host-side max(seq_lens) (avoids sync)
    workspace: Optional[object] = None
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
