"""Pieces that several model families share."""
from __future__ import annotations

from typing import Tuple

import torch.nn as nn


def round_up(n: int, m: int) -> int:
    return -(-n // m) * m


class Float32Kept(nn.Module):
    """Small tensors that keep their 32 (or 64) bits through .to(bfloat16):
    the kernels use them that way (norm weights, mixing coefficients, decays,
    rotation frequencies)."""
    kept: Tuple[str, ...] = ()

    def _apply(self, fn, recurse=True):
        held = {n: getattr(self, n).data for n in self.kept
                if getattr(self, n) is not None}
        super()._apply(fn, recurse)
        for n, t in held.items():
            cur = getattr(self, n)
            cur.data = t.to(cur.device)
        return self
