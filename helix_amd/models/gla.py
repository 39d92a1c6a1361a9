"""Gated linear attention: a linear recurrence over a [dim, vdim] matrix per
head with a decay per key channel and token,

    S <- diag(alpha) S + k v^T,  o = S^T q,
    alpha = sigmoid(a2 a1 h + b)^(1/tau),

each head's o RMS-normed and gated by silu(g).

or with a constant decay per head ("lightning"),

    S <- decay S + silu(k) silu(v)^T,  o = S^T silu(q),

all heads' o RMS-normed together and gated by sigmoid(g).

Single tokens do all but that common norm in one launch. Prompts run chunks
of 64 tokens in the dual form on MFMA and carry the state from chunk to chunk
in registers.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Tuple

import torch
import torch.nn as nn

from helix_amd.models.base import Float32Kept, round_up
from helix_amd.models.meta import MixedMeta, StateLayer
from helix_amd.ops import gated


@dataclass(frozen=True)
class GLASpec:
    heads: int
    dim: int                     # query / key size per head
    vdim: int
    tau: float
    rank: int                    # of the decays' projection

    @classmethod
    def from_json(cls, m: dict, rank: int) -> "GLASpec":
        return cls(heads=m["heads"], dim=m["dim"], vdim=m["vdim"],
                   tau=float(m["tau"]), rank=rank)

    def inputs(self) -> list:
        """(checkpoint name, columns) of what is projected from a row."""
        k, v = self.heads * self.dim, self.heads * self.vdim
        return [("q", k), ("k", k), ("v", v), ("g", v), ("a1", self.rank)]

    bias = shared_kv = False

    @property
    def out_size(self) -> int:
        return self.heads * self.vdim

    def cache_layer(self) -> StateLayer:
        return StateLayer((((self.heads, self.dim, round_up(self.vdim, 4)),
                            torch.float32),))

    def activation_floats(self) -> int:
        """Per prompt token: projections, results, and the chunks' operands
        (two terms of queries, keys and scores)."""
        k, v = self.heads * self.dim, self.heads * self.vdim
        return (6 * k + 5 * v + 2 * self.heads * gated.GLA_CHUNK) // 2

    def other_weights(self) -> int:
        return self.heads * self.dim * (self.rank + 1)


class GatedLinearAttention(Float32Kept):
    """Everything between the fused projections; at: first column of each
    input in the fused projection."""
    kept = ("a2_b", "norm_w")

    def __init__(self, spec: GLASpec, at: dict, eps: float,
                 out_scale: float = 1.0):
        super().__init__()
        self.spec = spec
        n = spec.heads * spec.dim
        self.params = gated.GLAParams(
            spec.heads, spec.dim, spec.vdim, spec.rank, at["q"], at["k"],
            at["v"], at["g"], at["a1"], spec.tau, eps, out_scale)
        self.a2 = nn.Parameter(torch.zeros(n, round_up(spec.rank, 32)))
        self.a2_b = nn.Parameter(torch.zeros(n))
        self.norm_w = nn.Parameter(torch.ones(spec.vdim))

    @property
    def weights(self) -> gated.GLAWeights:
        return gated.GLAWeights(self.a2, self.a2_b, self.norm_w)

    def scratch_floats(self, max_batch: int, max_len: int) -> int:
        return 0

    def forward(self, out, z, cache, meta, tables=None):
        p, w, (state,) = self.params, self.weights, cache
        if isinstance(meta, MixedMeta):
            n, d = meta.num_decode, meta.decode
            gated.gla_step(out[:n], z[:n], p, w, state, d.state_slots,
                           d.positions)
            gated.gla_prompt(out[n:], z[n:], p, w, state, meta.prefill)
        elif meta.is_prefill:
            gated.gla_prompt(out, z, p, w, state, meta)
        else:
            gated.gla_step(out, z, p, w, state, meta.state_slots,
                           meta.positions)

    def targets(self, prefix: str) -> dict:
        s = self.spec
        return {
            prefix + "a2": self.a2.data[:, :s.rank],
            prefix + "a2.b": self.a2_b.data,
            prefix + "norm": self.norm_w.data,
        }


@dataclass(frozen=True)
class LightningSpec:
    heads: int
    dim: int                     # query / key size per head
    vdim: int
    decay: Tuple[float, ...]     # per head

    def __post_init__(self):
        if len(self.decay) != self.heads or \
                not all(0 <= a <= 1 for a in self.decay):
            raise ValueError(f"decays {self.decay} of {self.heads} heads")

    @classmethod
    def from_json(cls, m: dict) -> "LightningSpec":
        return cls(heads=m["heads"], dim=m["dim"], vdim=m["vdim"],
                   decay=tuple(float(a) for a in m["decay"]))

    def inputs(self) -> list:
        k, v = self.heads * self.dim, self.heads * self.vdim
        return [("q", k), ("k", k), ("v", v), ("g", v)]

    bias = shared_kv = False

    @property
    def out_size(self) -> int:
        return self.heads * self.vdim

    def cache_layer(self) -> StateLayer:
        return StateLayer((((self.heads, self.dim, round_up(self.vdim, 4)),
                            torch.float32),))

    def activation_floats(self) -> int:
        k, v = self.heads * self.dim, self.heads * self.vdim
        return (6 * k + 5 * v + 2 * self.heads * gated.GLA_CHUNK) // 2

    def other_weights(self) -> int:
        return self.out_size


class LightningAttention(Float32Kept):
    """Everything between the fused projections; at: first column of each
    input in the fused projection."""
    kept = ("decay", "log_decay", "norm_w")

    def __init__(self, spec: LightningSpec, at: dict, eps: float,
                 out_scale: float = 1.0):
        super().__init__()
        if out_scale != 1.0:
            raise ValueError("lightning attention has no output scale")
        self.spec = spec
        self.params = gated.DecayParams(
            spec.heads, spec.dim, spec.vdim, at["q"], at["k"], at["v"],
            at["g"], eps)
        self.register_buffer("decay", torch.tensor(spec.decay),
                             persistent=False)
        # a decay of 0 leaves nothing after one token, as 2^-1000 does
        self.register_buffer("log_decay", torch.tensor(
            [math.log2(a) if a > 0 else -1000.0 for a in spec.decay]),
            persistent=False)
        self.norm_w = nn.Parameter(torch.ones(spec.out_size))

    @property
    def weights(self) -> gated.DecayWeights:
        return gated.DecayWeights(self.decay, self.log_decay, self.norm_w)

    def scratch_floats(self, max_batch: int, max_len: int) -> int:
        return 0

    def forward(self, out, z, cache, meta, tables=None):
        p, w, (state,) = self.params, self.weights, cache
        if isinstance(meta, MixedMeta):
            n, d = meta.num_decode, meta.decode
            gated.decay_step(out[:n], z[:n], p, w, state, d.state_slots,
                             d.positions)
            gated.decay_prompt(out[n:], z[n:], p, w, state, meta.prefill)
        elif meta.is_prefill:
            gated.decay_prompt(out, z, p, w, state, meta)
        else:
            gated.decay_step(out, z, p, w, state, meta.state_slots,
                             meta.positions)

    def targets(self, prefix: str) -> dict:
        return {prefix + "norm": self.norm_w.data}
