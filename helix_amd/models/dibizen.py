"""Dibizen: softmax attention, selective scans and lightning attention in
layers of any order, each with a mixture of experts, over several residual
streams.

With the streams x_1 .. x_S, for a sublayer (mixer, then feed-forward) and its
coefficients in, out, mix:

    y   = sublayer(norm(sum_s in[s] x_s))
    x_t <- sum_s mix[s, t] x_s + out[t] y

norm is tanh(alpha u) w + b. All streams start as token plus position
embedding; their sum goes to the final norm, the logits are soft-capped. An
attention layer may read the keys and values of an earlier one.

MI355X layout: the streams are fp32 [T, S, W]; one launch takes a sublayer's
result into all of them and norms what the next one reads. A mixture's
experts are two launches of one product each, and their weighted sum is taken
where the streams are updated.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import List, Optional, Tuple

import torch
import torch.nn as nn

from helix_amd.models.base import Float32Kept
from helix_amd.models.gla import LightningSpec
from helix_amd.models.llama import HLinear
from helix_amd.models.mixer_group import GroupSpec, Member, MixerGroup
from helix_amd.models.moe import Mixture, MixtureSpec
from helix_amd.models.rotary_attention import (AttnSpec, QueryTemperature,
                                               RotaryTables)
from helix_amd.models.selective import SelectiveSpec
from helix_amd.ops import gated, routed
from helix_amd.ops.routed import RouterParams


def attention(kv_from: Optional[int] = None, **sizes) -> AttnSpec:
    return AttnSpec(gate=True, shared_kv=kv_from is not None, **sizes)


def _attention(m: dict) -> AttnSpec:
    return attention(
        m.get("kv_from"), heads=m["heads"], kv_heads=m["kv_heads"],
        dim=m["dim"], vdim=m["vdim"], scale=float(m["scale"]),
        q_temp=QueryTemperature.from_json(m.get("q_temp")))


MIXERS = {"attention": _attention, "lightning": LightningSpec.from_json,
          "mamba1": SelectiveSpec.from_json}


@dataclass(frozen=True)
class LayerSpec:
    mixer: GroupSpec
    ff: Optional[MixtureSpec] = None
    kv_from: Optional[int] = None    # layer whose keys and values it reads

    @classmethod
    def of(cls, mixer, ff=None, kv_from=None) -> "LayerSpec":
        return cls(GroupSpec((Member(mixer),)), ff, kv_from)


@dataclass(frozen=True)
class DibizenConfig:
    name: str
    vocab_size: int
    hidden_size: int
    layers: Tuple[LayerSpec, ...]
    streams: int
    max_position: int            # rows of the position table
    logit_softcap: float
    norm_eps: float = 1e-5

    def __post_init__(self):
        if not 1 <= self.streams <= 8:
            raise ValueError(f"{self.streams} residual streams")
        if not self.logit_softcap > 0:
            raise ValueError(f"logit softcap {self.logit_softcap}")
        for i, l in enumerate(self.layers):
            if l.kv_from is None:
                continue
            src = self.layers[l.kv_from] if 0 <= l.kv_from < i else None
            a, b = l.mixer.members[0].spec, \
                src and src.mixer.members[0].spec
            if not isinstance(b, AttnSpec) or b.shared_kv or \
                    (a.kv_heads, a.dim, a.vdim) != (b.kv_heads, b.dim,
                                                    b.vdim):
                raise ValueError(f"layer {i} cannot read the keys and values "
                                 f"of layer {l.kv_from}")

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @property
    def position_limit(self) -> int:
        """Longest sequence: positions have learned vectors."""
        return self.max_position

    def kv_layers(self, tp_size: int = 1) -> list:
        return [c for l in self.layers for c in l.mixer.cache_layers()]

    def cache_entries(self) -> List[int]:
        """The cache entry of every layer, its own or the one it reads."""
        out, n = [], 0
        for l in self.layers:
            if l.kv_from is not None:
                out.append(out[l.kv_from])
            else:
                out.append(n)
                n += 1
        return out

    def num_weights(self) -> Tuple[int, int]:
        """(embeddings and head, per-layer total) parameter counts."""
        W = self.hidden_size
        n = sum(l.mixer.num_weights(W) + (l.ff.num_weights(W) if l.ff else 0)
                for l in self.layers)
        return (2 * self.vocab_size + self.max_position) * W, n

    def activation_bytes(self, tokens: int) -> int:
        """The streams and the widest layer's buffers."""
        W = self.hidden_size
        wide = max(l.mixer.activation_floats()
                   + (l.ff.activation_floats(W) if l.ff else 0)
                   for l in self.layers)
        return tokens * 4 * ((self.streams + 2) * W + 2 * wide)

    @classmethod
    def from_json(cls, d: dict, name: str = "dibizen") -> "DibizenConfig":
        layers = []
        for i, l in enumerate(d["layers"]):
            if l["type"] not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {l['type']!r}")
            mlp = l.get("mlp")
            if mlp is not None and mlp["kind"] != "moe":
                raise ValueError(f"layer {i}: unknown feed-forward "
                                 f"{mlp['kind']!r}")
            layers.append(LayerSpec.of(
                MIXERS[l["type"]](l["mixer"]),
                None if mlp is None else MixtureSpec.from_json(mlp),
                l["mixer"].get("kv_from")))
        return cls(
            name=name, vocab_size=d["vocab"], hidden_size=d["width"],
            layers=tuple(layers), streams=d["streams"],
            max_position=d["max_positions"],
            logit_softcap=float(d["logit_softcap"]),
            norm_eps=float(d["norm"]["eps"]))


def _preset(name, vocab, width, heads, ff, experts, top, blocks):
    """`blocks` times attention, selective scan, lightning attention and an
    attention layer that reads the first one's keys and values."""
    D = 128
    sizes = dict(heads=heads, kv_heads=heads // 4, dim=D, vdim=D,
                 scale=D ** -0.5, q_temp=QueryTemperature(0.1, 4096))
    moe = MixtureSpec(ff, RouterParams(experts, top, identity=experts // 8,
                                       groups=experts // 8, keep=4))
    layers = []
    for b in range(blocks):
        layers += [
            LayerSpec.of(attention(**sizes), moe),
            LayerSpec.of(SelectiveSpec(2 * width, 16, 4, width // 16), moe),
            LayerSpec.of(LightningSpec(heads, D, D, tuple(
                1 - 2.0 ** (-5 - 8 * h / heads) for h in range(heads))), moe),
            LayerSpec.of(attention(4 * b, **sizes), moe, 4 * b)]
    return DibizenConfig(name=name, vocab_size=vocab, hidden_size=width,
                         layers=tuple(layers), streams=4, max_position=32768,
                         logit_softcap=30.0)


PRESETS = {
    # 8B-class widths; 28B weights, 5B of them active per token
    "dibizen-28b": _preset("dibizen-28b", 128256, 4096, 32, 1536, 64, 8, 8),
    "dibizen-3b": _preset("dibizen-3b", 32000, 2048, 16, 768, 64, 8, 3),
    # mixed layers for CPU tests and smoke runs
    "tiny-dibizen": DibizenConfig(
        name="tiny-dibizen", vocab_size=512, hidden_size=128, layers=(
            LayerSpec.of(LightningSpec(3, 24, 20, (0.9, 0.5, 0.99)),
                         MixtureSpec(48, RouterParams(6, 2, 2, 4, 2))),
            LayerSpec.of(attention(
                heads=4, kv_heads=2, dim=32, vdim=24, scale=0.2,
                q_temp=QueryTemperature(0.4, 16)), None),
            LayerSpec.of(SelectiveSpec(160, 12, 3, 10),
                         MixtureSpec(64, RouterParams(5, 3))),
            LayerSpec.of(attention(
                1, heads=6, kv_heads=2, dim=32, vdim=24, scale=0.3),
                MixtureSpec(40, RouterParams(7, 3, 1, 2, 1)), 1),
        ), streams=2, max_position=512, logit_softcap=20.0),
}


class HyperNorm(Float32Kept):
    """What surrounds a sublayer: how it reads the streams, its norm, and how
    its result goes back."""
    kept = ("into", "out", "mix", "alpha", "w", "b")

    def __init__(self, streams: int, width: int, back: bool = True):
        super().__init__()
        ones = torch.ones(streams)
        self.into = nn.Parameter(ones.clone() if not back
                                 else ones / streams)
        self.out = nn.Parameter(ones.clone()) if back else None
        self.mix = nn.Parameter(torch.eye(streams)) if back else None
        self.alpha = nn.Parameter(torch.ones(1))
        self.w = nn.Parameter(torch.ones(width))
        self.b = nn.Parameter(torch.zeros(width))

    @property
    def norm(self) -> routed.TanhNorm:
        return routed.TanhNorm(self.alpha, self.w, self.b)

    @property
    def back(self) -> routed.Return:
        return routed.Return(self.mix, self.out)

    def targets(self, norm: str, hyper: Optional[str] = None) -> dict:
        out = {norm: self.w.data, norm + ".b": self.b.data,
               norm + ".alpha": self.alpha.data[0]}
        if hyper is not None:
            out.update({hyper + ".in": self.into.data,
                        hyper + ".out": self.out.data,
                        hyper + ".mix": self.mix.data})
        return out


class DibizenLayer(nn.Module):
    def __init__(self, cfg: DibizenConfig, index: int):
        super().__init__()
        spec, W = cfg.layers[index], cfg.hidden_size
        self.mixer = MixerGroup(spec.mixer, W, cfg.norm_eps)
        self.around = nn.ModuleList([HyperNorm(cfg.streams, W)])
        self.ff = None
        if spec.ff is not None:
            self.ff = Mixture(spec.ff, W)
            self.around.append(HyperNorm(cfg.streams, W))

    def targets(self, prefix: str) -> dict:
        out = self.mixer.targets(prefix + "mix.")
        if self.ff is not None:
            out.update(self.ff.targets(prefix + "mlp."))
        for q, a in enumerate(self.around, 1):
            out.update(a.targets(f"{prefix}norm{q}", f"{prefix}hc{q}"))
        return out


class DibizenForCausalLM(nn.Module):
    paged_prefill = True         # prompts attend through the paged cache
    extension = "_C_gated,_C_routed"     # native libraries of its kernels

    def __init__(self, cfg: DibizenConfig, tp_size: int = 1,
                 tp_rank: int = 0):
        if tp_size != 1:
            raise ValueError("dibizen runs on one GPU: all heads of a token "
                             "are normed together (tp_size must be 1)")
        super().__init__()
        self.cfg = cfg
        self.tp_size, self.tp_rank = tp_size, tp_rank
        W = cfg.hidden_size
        self.embed_tokens = nn.Embedding(cfg.vocab_size, W)
        self.places = nn.Parameter(torch.empty(cfg.max_position, W))
        self.layers = nn.ModuleList(
            [DibizenLayer(cfg, i) for i in range(cfg.num_layers)])
        self.final = HyperNorm(cfg.streams, W, back=False)
        self.lm_head = HLinear(W, cfg.vocab_size, bias=False)
        self.cache_at = cfg.cache_entries()
        # optional list receiving the streams' sum after every layer
        self.layer_tap: Optional[list] = None

    def decode_workspace(self, max_batch: int, max_len: int, device):
        """Flat fp32 scratch, enough for any layer at any batch size."""
        n = max(l.mixer.scratch_floats(max_batch, max_len)
                for l in self.layers)
        return torch.empty(2 * n, dtype=torch.float32, device=device)

    @torch.inference_mode()
    def forward(self, input_ids: torch.Tensor, kv_caches, meta):
        emb, cfg = self.embed_tokens.weight, self.cfg
        tables = RotaryTables(meta.positions)
        x = torch.empty(input_ids.shape[0], cfg.streams, cfg.hidden_size,
                        dtype=torch.float32, device=emb.device)
        around = [a for l in self.layers for a in l.around] + [self.final]
        at = 0                               # what the next sublayer reads by
        h = routed.hyper_embed(x, input_ids, meta.positions, emb,
                               self.places, around[0].into, around[0].norm)

        def back(y, tap=None):
            nonlocal at
            at += 1
            nxt = around[at]
            return routed.hyper_step(x, y, around[at - 1].back, nxt.into,
                                     nxt.norm, tap)

        for i, layer in enumerate(self.layers):
            tap = None
            if self.layer_tap is not None:
                tap = torch.empty(x.shape[0], x.shape[2], device=x.device)
                self.layer_tap.append(tap)
            y = layer.mixer(h, [kv_caches[self.cache_at[i]]], meta, tables)
            if layer.ff is not None:
                h = back(y)
                y = layer.ff(h)
            h = back(y, tap)
        return h

    @torch.inference_mode()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """fp32, soft-capped."""
        z = gated.project32(hidden, self.lm_head.weight)
        return routed.softcap(z, self.cfg.logit_softcap)

    # ------------------------------------------------------------------
    def checkpoint_targets(self) -> dict:
        """Checkpoint tensor name -> the view or Placement it is loaded
        into."""
        out = {"embed": self.embed_tokens.weight.data,
               "pos": self.places.data, "head": self.lm_head.weight.data}
        out.update(self.final.targets("final.norm"))
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
        S = self.cfg.streams

        def fill(dst, std, mean=0.0):
            dst.copy_(torch.randn(tuple(dst.shape), generator=g, device=dev)
                      * std + mean)

        for name, t in self.checkpoint_targets().items():
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("norm", "norm1", "norm2", "alpha", "out", "D"):
                fill(t, 0.05, 1.0)
            elif leaf == "in":
                fill(t, 0.05, 1.0 / S)
            elif name.endswith((".hc1.mix", ".hc2.mix")):
                t.copy_(torch.eye(S, device=dev) * 0.9 + 0.1 / S)
            elif leaf == "A_log":
                t.copy_(torch.rand(t.shape, generator=g, device=dev)
                        * math.log(16.0))
            elif name.endswith("dt.b"):
                fill(t, 0.5, -3.0)
            elif leaf == "conv":
                fill(t, t.shape[1] ** -0.5)
            elif leaf == "correction":
                fill(t, 0.01)
            else:
                fill(t, 0.02)
        return self

    def memory_bytes(self) -> int:
        return sum(p.numel() * p.element_size() for p in self.parameters())
