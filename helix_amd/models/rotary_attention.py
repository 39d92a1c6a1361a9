"""Attention over paged keys and values, with rotated positions or none.

Per head: score = (q . k) * scale over rotated q and k; weights are a softmax
or (sigmoid) each 1 / (1 + e^-(temp * score + bias)), not normalised. q and k
may be RMS-normed over their whole projections, values may be the unrotated
keys, and may travel rotated: cached turned by their position, results turned
back by the query's. A query may have a temperature that grows with its
position, results a gate per value; a layer without projections of its own
for keys and values reads those of another layer's cache.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch
import torch.nn as nn

from helix_amd import ops
from helix_amd.models.base import Float32Kept, round_up
from helix_amd.models.meta import KVLayer, MixedMeta
from helix_amd.ops import gated


@dataclass(frozen=True)
class HalvesRotary:
    """Dimension i of the first `dims` turns with i + dims/2; scaling as
    (factor, low, high, original), None = plain."""
    dims: int
    base: float
    scaling: Optional[tuple] = None

    def __post_init__(self):
        if self.dims % 2:
            raise ValueError(f"{self.dims} rotated dimensions")

    @classmethod
    def from_json(cls, d: Optional[dict]) -> Optional["HalvesRotary"]:
        if not d:
            return None
        s = d.get("scaling")
        return cls(int(d["dims"]), float(d["base"]), None if not s else tuple(
            float(s[k]) for k in ("factor", "low", "high", "original")))

    def frequencies(self) -> torch.Tensor:
        s = self.scaling
        return ops.banded_frequencies(
            self.dims, self.base, None if s is None else dict(
                zip(("factor", "low", "high", "original"), s)))


class RotaryTables:
    """What depends on a step's positions alone, made once for all layers
    that share it: cosines and sines, query temperatures."""

    def __init__(self, positions: torch.Tensor):
        self.positions = positions
        self.made: dict = {}

    def get(self, rotary: Optional[HalvesRotary], freqs):
        if rotary is None or not rotary.dims:
            return None
        if rotary not in self.made:
            self.made[rotary] = gated.rotary_table(self.positions, freqs)
        return self.made[rotary]

    def temperature(self, t: Optional["QueryTemperature"]):
        if t is None:
            return None
        if t not in self.made:
            self.made[t] = gated.query_temperature(self.positions, t.coef,
                                                   t.every)
        return self.made[t]


@dataclass(frozen=True)
class QueryTemperature:
    """A query at position p is multiplied by
    1 + coef * ln(floor((p + 1) / every) + 1)."""
    coef: float
    every: float

    def __post_init__(self):
        if self.every <= 0:
            raise ValueError(f"query temperature every {self.every} tokens")

    @classmethod
    def from_json(cls, d: Optional[dict]) -> Optional["QueryTemperature"]:
        return None if not d else cls(float(d["coef"]), float(d["every"]))


@dataclass(frozen=True)
class AttnSpec:
    heads: int
    kv_heads: int
    dim: int                     # query / key size per head
    vdim: int
    scale: float
    rotary: Optional[HalvesRotary] = None
    sigmoid: bool = False        # with a temperature and a bias per head
    tied_values: bool = False    # values are the unrotated keys
    bias: bool = False           # in the projections
    qk_norm: bool = False        # over the whole projections
    turn_values: bool = False
    q_temp: Optional[QueryTemperature] = None
    gate: bool = False           # sigmoid per value on the results
    shared_kv: bool = False      # no keys and values of its own

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads over {self.kv_heads} "
                             "key/value heads")
        if self.shared_kv and (self.tied_values or self.qk_norm):
            raise ValueError("shared keys and values have no projections "
                             "to tie or to norm")
        if self.tied_values and self.dim != self.vdim:
            raise ValueError(f"keys of {self.dim} as values of {self.vdim}")
        if self.rotary is not None and self.rotary.dims > self.dim:
            raise ValueError(f"{self.rotary.dims} rotated dimensions of "
                             f"{self.dim}")
        if self.value_rotary is not None and self.vdim % 2:
            raise ValueError(f"values of {self.vdim} cannot turn in pairs")

    @property
    def value_rotary(self) -> Optional[HalvesRotary]:
        """All of a value, with the keys' base and no scaling."""
        if not self.turn_values or self.rotary is None:
            return None
        return HalvesRotary(self.vdim, self.rotary.base)

    def inputs(self) -> list:
        """(checkpoint name, columns) of what is projected from a row."""
        out = [("q", self.heads * self.dim)]
        if not self.shared_kv:
            out.append(("k", self.kv_heads * self.dim))
            if not self.tied_values:
                out.append(("v", self.kv_heads * self.vdim))
        if self.gate:
            out.append(("g", self.out_size))
        return out

    @property
    def out_size(self) -> int:
        return self.heads * self.vdim

    def cache_layer(self) -> KVLayer:
        return KVLayer(self.kv_heads, round_up(self.dim, 8), self.vdim,
                       v_transposed=True)

    def activation_floats(self) -> int:
        """Per prompt token, half of a float per bf16 value."""
        return (sum(n for _, n in self.inputs()) + self.out_size
                + self.heads * self.dim) // 2

    def other_weights(self) -> int:
        return 0


class RotaryAttention(Float32Kept):
    """Everything between the fused projections; at: first column of each
    input in the fused projection."""
    kept = ("q_norm", "k_norm", "temp", "head_bias", "freqs", "value_freqs")

    def __init__(self, spec: AttnSpec, at: dict, eps: float,
                 out_scale: float = 1.0):
        super().__init__()
        self.spec, self.eps = spec, eps

        def vector(n, fill, on):
            return nn.Parameter(torch.full((n,), fill)) if on else None

        H, G, D = spec.heads, spec.kv_heads, spec.dim
        self.q_norm = vector(H * D, 1.0, spec.qk_norm)
        self.k_norm = vector(G * D, 1.0, spec.qk_norm)
        self.temp = vector(H, 1.0, spec.sigmoid)
        self.head_bias = vector(H, 0.0, spec.sigmoid)
        for name, rot in (("freqs", spec.rotary),
                          ("value_freqs", spec.value_rotary)):
            self.register_buffer(name, None if rot is None
                                 else rot.frequencies(), persistent=False)
        self._shape = dict(
            heads=H, kv_heads=G, dim=D, vdim=spec.vdim,
            dim_pad=round_up(D, 8), q_at=at["q"], k_at=at.get("k", -1),
            v_at=at.get("k" if spec.tied_values else "v", -1),
            scale=spec.scale, out_scale=out_scale, sigmoid=spec.sigmoid)
        self.gate_at = at.get("g", -1)

    @property
    def params(self) -> gated.AttnParams:
        return gated.AttnParams(temp=self.temp, bias=self.head_bias,
                                **self._shape)

    def scratch_floats(self, max_batch: int, max_len: int) -> int:
        p = self.params
        rows = {1, max_batch} | {2 ** i for i in range(12)
                                 if 2 ** i < max_batch}
        return max(gated.attn_scratch_floats(r, p, n)
                   for r in rows for n in (max_len, 512))

    def forward(self, out, z, kv_cache, meta, tables: RotaryTables):
        p, s = self.params, self.spec
        vcs = tables.get(s.value_rotary, self.value_freqs)
        q = gated.attn_epilogue(z, p, kv_cache, meta.slot_mapping,
                                tables.get(s.rotary, self.freqs), vcs,
                                self.q_norm, self.k_norm, self.eps)
        # one entry per row of the batch, as out and q
        by_row = dict(vcs=vcs, row_scale=tables.temperature(s.q_temp),
                      gate=z[:, self.gate_at:self.gate_at + s.out_size]
                      if s.gate else None)

        def rows(of: slice) -> dict:
            return {k: None if t is None else t[of]
                    for k, t in by_row.items()}

        if isinstance(meta, MixedMeta):
            n = meta.num_decode
            self._rows(out[:n], q[:n], p, kv_cache, meta.decode,
                       rows(slice(0, n)))
            gated.attn_prompt(out[n:], q[n:], p, kv_cache, meta.prefill,
                              **rows(slice(n, None)))
        elif meta.is_prefill:
            gated.attn_prompt(out, q, p, kv_cache, meta, **by_row)
        else:
            self._rows(out, q, p, kv_cache, meta, by_row)

    @staticmethod
    def _rows(out, q, p, kv_cache, meta, by_row):
        gated.attn_rows(out, q, p, kv_cache, meta.block_tables,
                        meta.seq_lens, meta.max_len,
                        workspace=meta.workspace, **by_row)

    def targets(self, prefix: str) -> dict:
        named = {"q.norm": self.q_norm, "k.norm": self.k_norm,
                 "temp": self.temp, "pb": self.head_bias}
        return {prefix + n: t.data for n, t in named.items()
                if t is not None}
