"""Mamba-2 mixer: a per-head linear recurrence over a [state, vdim] matrix
with a scalar decay per token, after a short causal convolution.

Single tokens update the state in one launch (convolution, step size,
recurrence, gate). Prompts run chunks of 64 tokens in the dual form on MFMA
and carry the state from chunk to chunk in registers."""
from __future__ import annotations

from dataclasses import dataclass

import torch
import torch.nn as nn

from helix_amd.engine.weights import Placement
from helix_amd.models.base import Float32Kept, round_up
from helix_amd.models.llama import HLinear
from helix_amd.models.meta import MixedMeta, StateLayer
from helix_amd.ops import hybrid


@dataclass(frozen=True)
class SSMSpec:
    heads: int
    vdim: int                    # value size per head
    state: int                   # state size per head
    groups: int                  # groups of heads that share B and C
    conv: int                    # convolution taps
    norm_groups: int

    def __post_init__(self):
        if self.heads % self.groups:
            raise ValueError(f"{self.heads} heads in {self.groups} groups")
        if self.inner % self.norm_groups:
            raise ValueError(f"{self.inner} values in {self.norm_groups} "
                             "norm groups")

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        return self.inner + 2 * self.groups * self.state

    @classmethod
    def from_json(cls, m: dict) -> "SSMSpec":
        return cls(**{k: int(m[k]) for k in (
            "heads", "vdim", "state", "groups", "conv", "norm_groups")})

    def cache_layer(self) -> StateLayer:
        """Ring of the convolution's last inputs, and the state."""
        return StateLayer((
            ((self.conv, self.channels), None),
            ((self.heads, self.state, self.vdim), torch.float32)))

    def num_weights(self, width: int) -> int:
        return (width * (2 * self.inner + self.channels + self.heads)
                + self.channels * (self.conv + 1) + self.inner)

    def activation_floats(self) -> int:
        return (3 * self.inner + 3 * self.channels) // 2


class Mamba2Mixer(Float32Kept):
    kept = ("conv_w", "conv_b", "dt_bias", "A_log", "D", "norm_w")

    def __init__(self, spec: SSMSpec, width: int, eps: float):
        super().__init__()
        self.spec, self.eps = spec, eps
        xbc_at = round_up(spec.inner, 8)
        dt_at = round_up(xbc_at + spec.channels, 8)
        self.params = hybrid.SSMParams(
            spec.heads, spec.vdim, spec.state, spec.groups, spec.conv,
            z_at=0, xbc_at=xbc_at, dt_at=dt_at)
        self.in_proj = HLinear(width, round_up(dt_at + spec.heads, 64),
                               bias=False)
        self.in_proj.weight.data.zero_()
        self.o_proj = HLinear(spec.inner, width, bias=False)
        self.conv_w = nn.Parameter(torch.zeros(spec.channels, spec.conv))
        self.conv_b = nn.Parameter(torch.zeros(spec.channels))
        self.dt_bias = nn.Parameter(torch.zeros(spec.heads))
        self.A_log = nn.Parameter(torch.zeros(spec.heads))
        self.D = nn.Parameter(torch.ones(spec.heads))
        self.norm_w = nn.Parameter(torch.ones(spec.inner))

    def scratch_floats(self, max_batch: int, max_len: int) -> int:
        return 0

    def forward(self, h, cache, meta):
        z = self.in_proj(h)
        w = hybrid.SSMWeights(self.conv_w, self.conv_b, self.dt_bias,
                              self.A_log, self.D)
        y = torch.empty(h.shape[0], self.spec.inner, dtype=h.dtype,
                        device=h.device)
        if isinstance(meta, MixedMeta):
            n = meta.num_decode
            hybrid.ssm_step(y[:n], z[:n], self.params, w, cache,
                            meta.decode.state_slots, meta.decode.positions)
            hybrid.ssm_prompt(y[n:], z[n:], self.params, w, cache,
                              meta.prefill)
        elif meta.is_prefill:
            hybrid.ssm_prompt(y, z, self.params, w, cache, meta)
        else:
            hybrid.ssm_step(y, z, self.params, w, cache, meta.state_slots,
                            meta.positions)
        return self.o_proj(hybrid.group_rms_norm(y, self.spec.norm_groups,
                                                 self.norm_w, self.eps))

    def targets(self, prefix: str) -> dict:
        s, p, w = self.spec, self.params, self.in_proj.weight.data
        a, b = s.inner, s.inner + s.channels
        return {
            prefix + "in": Placement((b + s.heads, w.shape[1]), [
                (w[p.z_at:p.z_at + a], lambda t: t[:a]),
                (w[p.xbc_at:p.xbc_at + s.channels], lambda t: t[a:b]),
                (w[p.dt_at:p.dt_at + s.heads], lambda t: t[b:])]),
            prefix + "conv": self.conv_w.data,
            prefix + "conv.b": self.conv_b.data,
            prefix + "dt_bias": self.dt_bias.data,
            prefix + "A_log": self.A_log.data,
            prefix + "D": self.D.data,
            prefix + "norm": self.norm_w.data,
            prefix + "o": self.o_proj.weight.data,
        }
