"""Selective scan mixer (Mamba-1): a short causal convolution, then a linear
recurrence per channel and state whose step sizes, inputs and readouts depend
on the token,

    x = silu(conv(x));  [dt | B | C] = W_x x;  dt = softplus(W_dt dt + b)
    S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n
    y_c = (sum_n S[c, n] C_n + D_c x_c) silu(z_c)
"""
from __future__ import annotations

import math
from dataclasses import dataclass

import torch
import torch.nn as nn

from helix_amd.engine.weights import Placement
from helix_amd.models.base import Float32Kept, round_up
from helix_amd.models.meta import MixedMeta, StateLayer
from helix_amd.ops import routed


@dataclass(frozen=True)
class SelectiveSpec:
    inner: int                   # channels
    state: int                   # per channel
    conv: int                    # convolution taps
    dt_rank: int

    def __post_init__(self):
        # what the kernels hold in registers, and tokens of a block
        if not (1 <= self.state <= 128 and 1 <= self.conv <= 33):
            raise ValueError(f"state of {self.state}, {self.conv} taps")

    @classmethod
    def from_json(cls, m: dict) -> "SelectiveSpec":
        return cls(**{k: int(m[k]) for k in ("inner", "state", "conv",
                                             "dt_rank")})

    def inputs(self) -> list:
        return [("in", 2 * self.inner)]

    bias = shared_kv = False

    @property
    def out_size(self) -> int:
        return self.inner

    def cache_layer(self) -> StateLayer:
        """Ring of the convolution's last inputs, and the state."""
        return StateLayer((
            ((self.conv, self.inner), None),
            ((self.state, self.inner), torch.float32)))

    def activation_floats(self) -> int:
        """Per prompt token: x, z, the convolved x and y in half a float
        each, step sizes, B and C in fp32."""
        return 3 * self.inner + 2 * self.state + self.dt_rank

    def other_weights(self) -> int:
        return self.inner * (2 * self.dt_rank + 3 * self.state + self.conv
                             + 3)


class SelectiveScan(Float32Kept):
    """Everything between the input projection and the output projection;
    at: first column of each input in the fused projection."""
    kept = ("conv_w", "conv_b", "dt_b", "A", "D")

    def __init__(self, spec: SelectiveSpec, at: dict, eps: float,
                 out_scale: float = 1.0):
        super().__init__()
        if out_scale != 1.0:
            raise ValueError("the selective scan has no output scale")
        s = self.spec = spec
        I, N = s.inner, s.state
        b_at = round_up(s.dt_rank, 8)
        c_at = b_at + routed.state_columns(N)
        self.params = routed.ScanParams(
            I, N, s.conv, s.dt_rank, x_at=at["in"], z_at=at["in"] + I,
            b_at=b_at, c_at=c_at)
        self.x_w = nn.Parameter(torch.zeros(
            round_up(self.params.columns, 32), I))
        self.dt_w = nn.Parameter(torch.zeros(I, s.dt_rank))
        self.dt_b = nn.Parameter(torch.zeros(I))
        self.conv_w = nn.Parameter(torch.zeros(s.conv, I))
        self.conv_b = nn.Parameter(torch.zeros(I))
        self.A = nn.Parameter(torch.zeros(N, I))     # times log2(e)
        self.D = nn.Parameter(torch.ones(I))

    @property
    def weights(self) -> routed.ScanWeights:
        return routed.ScanWeights(self.conv_w, self.conv_b, self.x_w,
                                  self.dt_w, self.dt_b, self.A, self.D)

    def scratch_floats(self, max_batch: int, max_len: int) -> int:
        return 0

    def forward(self, out, z, cache, meta, tables=None):
        p, w = self.params, self.weights
        if isinstance(meta, MixedMeta):
            n, d = meta.num_decode, meta.decode
            routed.selective_step(out[:n], z[:n], p, w, cache, d.state_slots,
                                  d.positions)
            routed.selective_prompt(out[n:], z[n:], p, w, cache,
                                    meta.prefill)
        elif meta.is_prefill:
            routed.selective_prompt(out, z, p, w, cache, meta)
        else:
            routed.selective_step(out, z, p, w, cache, meta.state_slots,
                                  meta.positions)

    def targets(self, prefix: str) -> dict:
        s, p = self.spec, self.params
        R, N, x = s.dt_rank, s.state, self.x_w.data

        def transposed(dst, *shape):
            return Placement(shape, [(dst, lambda t: t.t())])

        return {
            prefix + "conv": transposed(self.conv_w.data, s.inner, s.conv),
            prefix + "conv.b": self.conv_b.data,
            prefix + "x": Placement((R + 2 * N, s.inner), [
                (x[:R], lambda t: t[:R]),
                (x[p.b_at:p.b_at + N], lambda t: t[R:R + N]),
                (x[p.c_at:p.c_at + N], lambda t: t[R + N:])]),
            prefix + "dt": self.dt_w.data,
            prefix + "dt.b": self.dt_b.data,
            prefix + "A_log": Placement((s.inner, N), [
                (self.A.data, lambda t: (-torch.exp(t.double())
                                         * math.log2(math.e)).t())]),
            prefix + "D": self.D.data,
        }
