"""Latent attention: keys and values of all heads come from one small latent
per token, and only the latent and one shared rotated key part are cached.

Per head, score = (q_n . W_uk c + q_r . k_r) * scale and value = W_uv c.
Two ways to run it:

- single rows move W_uk to the query (q_n^T W_uk c) and W_uv behind the
  softmax, so they read each cached row once for all heads;
- prompts spell out keys and values of the tokens they see with two GEMMs
  (fewer products per pair), the values already transposed for the kernel.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch
import torch.nn as nn

from helix_amd import ops
from helix_amd.engine.weights import Placement
from helix_amd.models.base import Float32Kept, round_up
from helix_amd.models.llama import HLinear
from helix_amd.models.meta import KVLayer, MixedMeta
from helix_amd.ops import hybrid


@dataclass(frozen=True)
class RotarySpec:
    """Interleaved pairs of the first `dims` dimensions; scaling as
    (factor, original, fast, slow), None = plain."""
    dims: int
    base: float
    scaling: Optional[tuple] = None

    @classmethod
    def from_json(cls, d: Optional[dict]) -> Optional["RotarySpec"]:
        if not d:
            return None
        s = d.get("scaling")
        return cls(int(d["dims"]), float(d["base"]), None if not s else tuple(
            float(s[k]) for k in ("factor", "original", "fast", "slow")))

    def frequencies(self):
        s = self.scaling
        return ops.yarn_frequencies(self.dims, self.base, None if s is None
                                    else dict(zip(("factor", "original",
                                                   "fast", "slow"), s)))


@dataclass(frozen=True)
class LatentSpec:
    heads: int
    dim: int                     # unrotated query / key size per head
    rot_dim: int                 # rotated size per head (keys: shared)
    vdim: int
    kv_rank: int                 # latent size
    scale: float
    window: int = 0              # visible tokens, own included (0 = all)
    rotary: Optional[RotarySpec] = None

    def __post_init__(self):
        r = self.rotary
        if r is not None and (r.dims % 2 or r.dims > self.rot_dim):
            raise ValueError(f"{r.dims} rotated dimensions of {self.rot_dim}")

    @classmethod
    def from_json(cls, m: dict) -> "LatentSpec":
        return cls(heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"],
                   vdim=m["vdim"], kv_rank=m["kv_rank"],
                   scale=float(m["scale"]),
                   window=int((m.get("mask") or {}).get("size") or 0),
                   rotary=RotarySpec.from_json(m.get("rot")))

    def cache_layer(self) -> KVLayer:
        return KVLayer(1, round_up(self.kv_rank, 8)
                       + round_up(self.rot_dim, 8), 0)

    def num_weights(self, width: int) -> int:
        H = self.heads
        return (width * (H * (self.dim + self.rot_dim + 1) + self.kv_rank
                         + self.rot_dim + H * self.vdim)
                + H * self.kv_rank * (self.dim + self.vdim))

    def activation_floats(self) -> int:
        """Per prompt token, half of a float per bf16 value."""
        H = self.heads
        return (H * (2 * self.dim + self.rot_dim + 2 * self.vdim)
                + 2 * self.kv_rank) // 2


class LatentAttention(Float32Kept):
    kept = ("kv_norm_w", "freqs")

    def __init__(self, spec: LatentSpec, width: int, eps: float):
        super().__init__()
        self.spec, self.eps = spec, eps
        H = spec.heads
        dp, rp, kp = (round_up(n, 8) for n in (spec.dim, spec.rot_dim,
                                               spec.kv_rank))
        # column starts in the fused projection, 16-byte aligned
        kv_at = H * (dp + rp)
        self.gate_at = kv_at + kp + rp
        self.in_proj = HLinear(width, round_up(self.gate_at + H, 64),
                               bias=False)
        self.o_proj = HLinear(H * spec.vdim, width, bias=False)
        # up-projections; uk also transposed per head for single rows
        self.uk = nn.Parameter(torch.zeros(H * dp, kp))
        self.ukt = nn.Parameter(torch.zeros(H, kp, dp))
        self.uv = nn.Parameter(torch.zeros(H * spec.vdim, kp))
        self.in_proj.weight.data.zero_()
        self.kv_norm_w = nn.Parameter(torch.ones(spec.kv_rank))
        freqs, amp = spec.rotary.frequencies() if spec.rotary is not None \
            else (None, 1.0)
        self.register_buffer("freqs", freqs, persistent=False)
        self._shape = dict(
            heads=H, dim=spec.dim, rot_dim=spec.rot_dim, vdim=spec.vdim,
            rank=spec.kv_rank, dim_pad=dp, rot_pad=rp, rank_pad=kp, q_at=0,
            kv_at=kv_at, scale=spec.scale, window=spec.window, amp=amp)

    @property
    def params(self) -> hybrid.LatentParams:
        return hybrid.LatentParams(freqs=self.freqs, **self._shape)

    def scratch_floats(self, max_batch: int, max_len: int) -> int:
        p = self.params
        rows = {1, max_batch} | {2 ** i for i in range(12)
                                 if 2 ** i < max_batch}
        return max(hybrid.latent_scratch_floats(r, p, n)
                   for r in rows for n in (max_len, 512))

    def forward(self, h, kv_cache, meta):
        p, cache = self.params, kv_cache[0]
        z = self.in_proj(h)
        hybrid.latent_epilogue(z, p, meta.positions, self.kv_norm_w, self.eps,
                               cache, meta.slot_mapping)
        out = torch.empty(h.shape[0], p.heads * p.vdim, dtype=h.dtype,
                          device=h.device)
        gate = z[:, self.gate_at:self.gate_at + p.heads]
        if isinstance(meta, MixedMeta):
            n = meta.num_decode
            self._rows(out[:n], z[:n], p, cache, meta.decode, gate[:n])
            self._prompt(out[n:], z[n:], p, cache, meta.prefill, gate[n:])
        elif meta.is_prefill:
            self._prompt(out, z, p, cache, meta, gate)
        else:
            self._rows(out, z, p, cache, meta, gate)
        return self.o_proj(out)

    def _rows(self, out, z, p, cache, meta, gate):
        hybrid.latent_attn_rows(out, z, p, cache, meta.block_tables,
                                meta.seq_lens, meta.max_len, self.uk,
                                self.ukt, self.uv, gate,
                                workspace=meta.workspace)

    def _prompt(self, out, z, p, cache, meta, gate):
        hybrid.latent_attn_prompt(out, z, p, cache, meta, self.uk, self.ukt,
                                  self.uv, gate)

    def targets(self, prefix: str) -> dict:
        s, p = self.spec, self.params
        H, D, R, K, W = (s.heads, s.dim, s.rot_dim, s.kv_rank,
                         self.in_proj.weight.shape[1])
        w = self.in_proj.weight.data
        q = w[:p.kv_at].view(H, p.head_cols, W)
        kv = w[p.kv_at:self.gate_at]
        uk = self.uk.data.view(H, p.dim_pad, p.rank_pad)
        return {
            prefix + "q": Placement((H * (D + R), W), [
                (q[:, :D], lambda t: t.view(H, D + R, W)[:, :D]),
                (q[:, p.dim_pad:p.dim_pad + R],
                 lambda t: t.view(H, D + R, W)[:, D:])]),
            prefix + "dkv": Placement((K + R, W), [
                (kv[:K], lambda t: t[:K]),
                (kv[p.rank_pad:p.rank_pad + R], lambda t: t[K:])]),
            prefix + "dkv.norm": self.kv_norm_w.data,
            prefix + "uk": Placement((H * D, K), [
                (uk[:, :D, :K], lambda t: t.view(H, D, K)),
                (self.ukt.data[:, :K, :D],
                 lambda t: t.view(H, D, K).transpose(1, 2))]),
            prefix + "uv": self.uv.data[:, :K],
            prefix + "g": w[self.gate_at:self.gate_at + H],
            prefix + "o": self.o_proj.weight.data,
        }
