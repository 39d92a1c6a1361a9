"""Pieces that several model families share."""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional, Tuple

import torch.nn as nn


def round_up(n: int, m: int) -> int:
    return -(-n // m) * m


@dataclass(frozen=True)
class LoopSpec:
    """Layers start .. stop-1 run `times` times in a row."""
    start: int
    stop: int
    times: int

    def check(self, layers: int):
        if not (0 <= self.start < self.stop <= layers and self.times >= 1):
            raise ValueError(f"loop {self} over {layers} layers")


@dataclass(frozen=True)
class LayerRun:
    layer: int
    loop_pass: int = -1          # number of the pass that begins here, or -1


def unroll(loop: Optional[LoopSpec], layers: int) -> List[LayerRun]:
    """The layers in the order they run."""
    l = loop or LoopSpec(0, 0, 0)
    out = [LayerRun(i) for i in range(l.start)]
    for t in range(l.times):
        out += [LayerRun(i, t if i == l.start else -1)
                for i in range(l.start, l.stop)]
    return out + [LayerRun(i) for i in range(l.stop, layers)]


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
