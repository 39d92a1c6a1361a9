"""Nibezen: latent-attention and Mamba-2 layers in any order, a stretch of
which runs several times in a row with the same weights.

A layer, with m the residual factor and s1, s2 its scale vectors:

    x <- x + m * s1 * mixer(norm(x))
    x <- x + m * s2 * ff(norm(x))          (SiLU-gated; may be missing)

Before every pass of the loop its step vector is added to x, before every
pass but the first the embedding as well. Each pass has a cache of its own,
so the cache has one entry per layer run, not per layer.

MI355X layout: the stream is fp32 and one launch does residual add, loop
entry and the next norm; q, latent and gate (or all of a Mamba-2 layer's
inputs) are one GEMM, gate and up of the feed-forward another.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import List, Optional, Tuple, Union

import torch
import torch.nn as nn

from helix_amd.models.base import (Float32Kept, LayerRun, LoopSpec, round_up,
                                   unroll)
from helix_amd.models.latent import LatentAttention, LatentSpec, RotarySpec
from helix_amd.models.llama import HLinear
from helix_amd.models.ssm import Mamba2Mixer, SSMSpec
from helix_amd.ops import hybrid

MIXERS = {"latent_attention": LatentSpec, "mamba2": SSMSpec}
MIXER_MODULES = {LatentSpec: LatentAttention, SSMSpec: Mamba2Mixer}


@dataclass(frozen=True)
class LayerSpec:
    mixer: Union[LatentSpec, SSMSpec]
    ff: int = 0                  # feed-forward size (0 = none)


@dataclass(frozen=True)
class NibezenConfig:
    name: str
    vocab_size: int
    hidden_size: int
    layers: Tuple[LayerSpec, ...]
    loop: Optional[LoopSpec] = None
    residual_mult: float = 1.0
    rms_norm_eps: float = 1e-6
    max_position: int = 1 << 20  # nothing in the design bounds it

    def __post_init__(self):
        if self.loop is not None:
            self.loop.check(len(self.layers))

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def runs(self) -> List[LayerRun]:
        """The layers in the order they run."""
        return unroll(self.loop, self.num_layers)

    def kv_layers(self, tp_size: int = 1) -> list:
        return [self.layers[r.layer].mixer.cache_layer()
                for r in self.runs()]

    def num_weights(self) -> Tuple[int, int]:
        """(embedding and head, per-layer total) parameter counts."""
        n = sum(l.mixer.num_weights(self.hidden_size)
                + 3 * self.hidden_size * l.ff for l in self.layers)
        return 2 * self.vocab_size * self.hidden_size, n

    def activation_bytes(self, tokens: int) -> int:
        """The stream and the widest layer's buffers."""
        wide = max(l.mixer.activation_floats() + 2 * l.ff
                   for l in self.layers)
        return tokens * 4 * (3 * self.hidden_size + 2 * wide)

    @classmethod
    def from_json(cls, d: dict, name: str = "nibezen") -> "NibezenConfig":
        layers = []
        for i, l in enumerate(d["layers"]):
            if l["type"] not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {l['type']!r}")
            mlp = l.get("mlp")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward "
                                 f"{mlp['kind']!r}")
            layers.append(LayerSpec(MIXERS[l["type"]].from_json(l["mixer"]),
                                    mlp["ff"] if mlp is not None else 0))
        loop = d.get("loop")
        return cls(
            name=name, vocab_size=d["vocab"], hidden_size=d["width"],
            layers=tuple(layers), loop=None if not loop else LoopSpec(
                loop["start"], loop["stop"], loop["times"]),
            residual_mult=float(d.get("residual_mult", 1.0)),
            rms_norm_eps=float(d["norm"]["eps"]))


def _hybrid(name, vocab, width, heads, rank, ff, window, ssm_heads, blocks,
            loop) -> NibezenConfig:
    """`blocks` times two attention layers and one Mamba-2 layer."""
    attn = LayerSpec(LatentSpec(
        heads=heads, dim=128, rot_dim=64, vdim=128, kv_rank=rank,
        scale=192 ** -0.5, window=window,
        rotary=RotarySpec(64, 500000.0, (4.0, 8192.0, 32.0, 1.0))), ff)
    ssm = LayerSpec(SSMSpec(heads=ssm_heads, vdim=64, state=128, groups=8,
                            conv=4, norm_groups=8), ff)
    return NibezenConfig(name=name, vocab_size=vocab, hidden_size=width,
                         layers=(attn, attn, ssm) * blocks, loop=loop,
                         residual_mult=0.5, max_position=32768)


PRESETS = {
    # 32 layer runs of an 8B-class decoder's sizes over 24 layers
    "nibezen-8b": _hybrid("nibezen-8b", 128256, 4096, 32, 512, 14336, 4096,
                          128, 8, LoopSpec(6, 10, 3)),
    "nibezen-1b": _hybrid("nibezen-1b", 32000, 2048, 16, 256, 5632, 2048,
                          64, 4, LoopSpec(3, 5, 3)),
    # mixed layers for CPU tests and smoke runs
    "tiny-nibezen": NibezenConfig(
        name="tiny-nibezen", vocab_size=512, hidden_size=128, layers=(
            LayerSpec(LatentSpec(5, 24, 8, 40, 48, 0.2, 40,
                                 RotarySpec(8, 1e4)), 192),
            LayerSpec(SSMSpec(4, 24, 40, 2, 3, 4), 0),
            LayerSpec(LatentSpec(3, 16, 16, 32, 32, 0.2, 0, RotarySpec(
                16, 1e5, (2.0, 256.0, 16.0, 1.0))), 320),
        ), loop=LoopSpec(0, 2, 2), residual_mult=0.8, rms_norm_eps=1e-5,
        max_position=512),
}


class NibezenLayer(Float32Kept):
    kept = ("norm1_w", "ls1", "norm2_w", "ls2")

    def __init__(self, cfg: NibezenConfig, index: int):
        super().__init__()
        spec, W = cfg.layers[index], cfg.hidden_size
        self.spec = spec
        self.mixer = MIXER_MODULES[type(spec.mixer)](spec.mixer, W,
                                                     cfg.rms_norm_eps)
        self.norm1_w = nn.Parameter(torch.ones(W))
        self.ls1 = nn.Parameter(torch.ones(W))
        self.norm2_w = self.ls2 = None
        if spec.ff:
            self.norm2_w = nn.Parameter(torch.ones(W))
            self.ls2 = nn.Parameter(torch.ones(W))
            self.up_at = round_up(spec.ff, 8)
            self.gate_up = HLinear(W, self.up_at + spec.ff, bias=False)
            self.gate_up.weight.data.zero_()
            self.down = HLinear(spec.ff, W, bias=False)

    def feed_forward(self, h):
        return self.down(hybrid.silu_mul(self.gate_up(h), self.up_at,
                                         self.spec.ff))

    def targets(self, prefix: str) -> dict:
        out = {prefix + "norm1": self.norm1_w.data,
               prefix + "ls1": self.ls1.data}
        out.update(self.mixer.targets(prefix + "mix."))
        if self.spec.ff:
            w, F = self.gate_up.weight.data, self.spec.ff
            out.update({prefix + "norm2": self.norm2_w.data,
                        prefix + "ls2": self.ls2.data,
                        prefix + "mlp.gate": w[:F],
                        prefix + "mlp.up": w[self.up_at:self.up_at + F],
                        prefix + "mlp.down": self.down.weight.data})
        return out


class NibezenForCausalLM(Float32Kept):
    kept = ("final_norm_w", "loop_step")
    paged_prefill = True         # prompts attend through the paged cache
    extension = "_C_hybrid"      # native library of its kernels

    def __init__(self, cfg: NibezenConfig, tp_size: int = 1,
                 tp_rank: int = 0):
        if tp_size != 1:
            raise ValueError("nibezen runs on one GPU: all heads of a token "
                             "share its latent (tp_size must be 1)")
        super().__init__()
        self.cfg = cfg
        self.tp_size, self.tp_rank = tp_size, tp_rank
        self.embed_tokens = nn.Embedding(cfg.vocab_size, cfg.hidden_size)
        self.layers = nn.ModuleList(
            [NibezenLayer(cfg, i) for i in range(cfg.num_layers)])
        self.loop_step = nn.Parameter(torch.zeros(
            cfg.loop.times, cfg.hidden_size)) if cfg.loop else None
        self.final_norm_w = nn.Parameter(torch.ones(cfg.hidden_size))
        self.lm_head = HLinear(cfg.hidden_size, cfg.vocab_size, bias=False)
        self.runs = cfg.runs()
        # optional list receiving the stream after every layer run
        self.layer_tap: Optional[list] = None

    def decode_workspace(self, max_batch: int, max_len: int, device):
        """Flat fp32 scratch, enough for any layer at any batch size."""
        n = max(l.mixer.scratch_floats(max_batch, max_len)
                for l in self.layers)
        return torch.empty(2 * n, dtype=torch.float32, device=device)

    def _entry(self, run: Optional[LayerRun], input_ids) -> dict:
        """What is added to the stream ahead of a layer run."""
        if run is None or run.loop_pass < 0:
            return {}
        add = {"step": self.loop_step[run.loop_pass]}
        if run.loop_pass > 0:
            add.update(ids=input_ids, embed=self.embed_tokens.weight)
        return add

    @torch.inference_mode()
    def forward(self, input_ids: torch.Tensor, kv_caches, meta):
        cfg, runs = self.cfg, self.runs
        eps, m = cfg.rms_norm_eps, cfg.residual_mult
        emb = self.embed_tokens.weight
        dtype = emb.dtype
        x = torch.empty(input_ids.shape[0], cfg.hidden_size,
                        dtype=torch.float32, device=emb.device)
        first = self._entry(runs[0], input_ids)
        h = hybrid.residual_norm(
            None, None, None, m, self.layers[runs[0].layer].norm1_w, eps,
            dtype, ids=input_ids, embed=emb, step=first.get("step"), x_out=x)
        for j, run in enumerate(runs):
            layer = self.layers[run.layer]
            nxt = runs[j + 1] if j + 1 < len(runs) else None
            y, ls = layer.mixer(h, kv_caches[j], meta), layer.ls1
            if layer.spec.ff:
                h = hybrid.residual_norm(x, y, ls, m, layer.norm2_w, eps,
                                         dtype, x_out=x)
                y, ls = layer.feed_forward(h), layer.ls2
            tap = None
            if self.layer_tap is not None:
                tap = torch.empty_like(x)
                self.layer_tap.append(tap)
            w = self.final_norm_w if nxt is None \
                else self.layers[nxt.layer].norm1_w
            h = hybrid.residual_norm(x, y, ls, m, w, eps, dtype, x_out=x,
                                     tap=tap, **self._entry(nxt, input_ids))
        return h

    @torch.inference_mode()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return self.lm_head(hidden)

    # ------------------------------------------------------------------
    def checkpoint_targets(self) -> dict:
        """Checkpoint tensor name -> the view or Placement it is loaded
        into."""
        out = {"embed": self.embed_tokens.weight.data,
               "head": self.lm_head.weight.data,
               "final.norm": self.final_norm_w.data}
        if self.loop_step is not None:
            out["loop.step"] = self.loop_step.data
        for i, l in enumerate(self.layers):
            out.update(l.targets(f"l{i}."))
        return out

    def optional_checkpoint_names(self) -> set:
        return set()

    @torch.inference_mode()
    def init_random(self, seed: int = 0):
        """Random weights with every mechanism active."""
        dev = self.embed_tokens.weight.device
        g = torch.Generator(device=dev).manual_seed(seed)

        def fill(dst, std, mean=0.0):
            dst.copy_(torch.randn(tuple(dst.shape), generator=g, device=dev)
                      * std + mean)

        for name, t in self.checkpoint_targets().items():
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("norm", "norm1", "norm2", "ls1", "ls2", "D"):
                fill(t, 0.05, 1.0)
            elif leaf == "A_log":
                t.copy_(torch.rand(t.shape, generator=g, device=dev)
                        * math.log(16.0))
            elif leaf == "dt_bias":
                fill(t, 0.5, -3.0)
            elif leaf == "conv":
                fill(t, t.shape[1] ** -0.5)
            else:
                fill(t, 0.02)
        return self

    def memory_bytes(self) -> int:
        return sum(p.numel() * p.element_size() for p in self.parameters())
