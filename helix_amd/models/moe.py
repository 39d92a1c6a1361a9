"""Mixture of experts as a feed-forward: a router in fp32 chooses a few
experts per token, limited to the best groups of them; some experts may be
identities. The result is left as the experts' rows with their weights, for
the residual stream to add up."""
from __future__ import annotations

from dataclasses import dataclass

import torch
import torch.nn as nn

from helix_amd.models.base import Float32Kept
from helix_amd.ops import gated, routed
from helix_amd.ops.routed import RouterParams


@dataclass(frozen=True)
class MixtureSpec:
    ff: int                      # of an expert: down(relu(up h)^2)
    router: RouterParams

    @classmethod
    def from_json(cls, d: dict) -> "MixtureSpec":
        r = d["router"]
        g = r.get("groups") or {"count": 1, "keep": 1}
        return cls(d["expert"]["ff"], RouterParams(
            experts=r["experts"], top=r["top"],
            identity=r.get("identity") or 0, groups=g["count"],
            keep=g["keep"]))

    def num_weights(self, width: int) -> int:
        r = self.router
        return 2 * r.experts * width * self.ff + r.outputs * (width + 1)

    def activation_floats(self, width: int) -> int:
        """Per token, half a float per bf16 value."""
        return self.router.top * (width + self.ff) // 2


class Mixture(Float32Kept):
    kept = ("correction",)

    def __init__(self, spec: MixtureSpec, width: int):
        super().__init__()
        self.spec = spec
        r = spec.router
        self.router = nn.Parameter(torch.zeros(r.outputs, width))
        self.correction = nn.Parameter(torch.zeros(r.outputs))
        self.ups = nn.Parameter(torch.empty(r.experts, spec.ff, width))
        self.downs = nn.Parameter(torch.empty(r.experts, width, spec.ff))

    def forward(self, h) -> routed.RoutedRows:
        return routed.expert_mixture(h, gated.project32(h, self.router),
                                     self.correction, self.ups, self.downs,
                                     self.spec.router)

    def targets(self, prefix: str) -> dict:
        out = {prefix + "router": self.router.data,
               prefix + "correction": self.correction.data}
        for e in range(self.spec.router.experts):
            out[f"{prefix}e{e}.up"] = self.ups.data[e]
            out[f"{prefix}e{e}.down"] = self.downs.data[e]
        return out
