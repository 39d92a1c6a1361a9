"""Mixers that read the same rows and whose scaled results add up: one fused
projection in, one out, whose accumulator does the addition.

A member is a spec (inputs(), out_size, bias, cache_layer(); shared_kv if it
has no cache of its own) with its module (forward(out, z, cache, meta, tables)
fills its columns of the buffer that
the output projection reads; its scale is applied there, in fp32).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Tuple, Union

import torch
import torch.nn as nn

from helix_amd.models.base import round_up
from helix_amd.models.gla import (GatedLinearAttention, GLASpec,
                                  LightningAttention, LightningSpec)
from helix_amd.models.llama import HLinear
from helix_amd.models.rotary_attention import AttnSpec, RotaryAttention
from helix_amd.models.selective import SelectiveScan, SelectiveSpec

MODULES = {AttnSpec: RotaryAttention, GLASpec: GatedLinearAttention,
           LightningSpec: LightningAttention, SelectiveSpec: SelectiveScan}
MixerSpec = Union[AttnSpec, GLASpec, LightningSpec, SelectiveSpec]


@dataclass(frozen=True)
class Member:
    spec: MixerSpec
    prefix: str = ""             # of its checkpoint names
    scale: float = 1.0


@dataclass(frozen=True)
class GroupSpec:
    members: Tuple[Member, ...]

    def __post_init__(self):
        if len(self.members) > 1 and any(m.spec.bias for m in self.members):
            raise ValueError("biases in a group of several mixers")

    @property
    def bias(self) -> bool:
        return any(m.spec.bias for m in self.members)

    def cache_layers(self) -> list:
        """Of the members that have a cache of their own."""
        return [m.spec.cache_layer() for m in self.members
                if not m.spec.shared_kv]

    def num_weights(self, width: int) -> int:
        return sum(width * (sum(n for _, n in m.spec.inputs())
                            + m.spec.out_size) + m.spec.other_weights()
                   for m in self.members)

    def activation_floats(self) -> int:
        return sum(m.spec.activation_floats() for m in self.members)


class MixerGroup(nn.Module):
    def __init__(self, spec: GroupSpec, width: int, eps: float):
        super().__init__()
        self.spec = spec
        # column starts in the fused projections, 16-byte aligned
        self.at: List[dict] = []
        self.out_at: List[int] = []
        n = k = 0
        for m in spec.members:
            at = {}
            for name, size in m.spec.inputs():
                at[name] = n
                n = round_up(n + size, 8)
            self.at.append(at)
            self.out_at.append(k)
            k = round_up(k + m.spec.out_size, 8)
        self.in_proj = HLinear(width, round_up(n, 64), bias=spec.bias)
        self.out_proj = HLinear(k, width, bias=spec.bias)
        for p in self.parameters():
            p.data.zero_()
        self.cores = nn.ModuleList(
            [MODULES[type(m.spec)](m.spec, at, eps, m.scale)
             for m, at in zip(spec.members, self.at)])

    def scratch_floats(self, max_batch: int, max_len: int) -> int:
        return max(c.scratch_floats(max_batch, max_len) for c in self.cores)

    def forward(self, h, caches, meta, tables):
        """caches: one entry per member, of its own or shared."""
        z = self.in_proj(h)
        width = self.out_proj.weight.shape[1]
        buf = torch.empty(h.shape[0], width, dtype=h.dtype, device=h.device)
        ends = self.out_at[1:] + [width]
        for m, core, cache, at, end in zip(self.spec.members, self.cores,
                                           caches, self.out_at, ends):
            stop = at + m.spec.out_size
            core(buf[:, at:stop], z, cache, meta, tables)
            if stop < end:
                buf[:, stop:end].zero_()
        return self.out_proj(buf)

    def targets(self, prefix: str) -> dict:
        w, o = self.in_proj.weight.data, self.out_proj.weight.data
        out = {}
        for m, core, at, o_at in zip(self.spec.members, self.cores, self.at,
                                     self.out_at):
            p = prefix + m.prefix
            for name, n in m.spec.inputs():
                a = at[name]
                out[p + name] = w[a:a + n]
                if m.spec.bias:
                    out[p + name + ".b"] = self.in_proj.bias.data[a:a + n]
            out[p + "o"] = o[:, o_at:o_at + m.spec.out_size]
            if m.spec.bias:
                out[p + "o.b"] = self.out_proj.bias.data
            out.update(core.targets(p))
        return out
