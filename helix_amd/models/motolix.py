"""Motolix: sigmoid attention, and softmax attention beside gated linear
attention, in layers of any order; a stretch of them may run several times in
a row with the same weights.

A layer, every norm a layer norm with bias:

    x <- x + post1(mixer(norm1(x)))
    x <- x + post2(down(gelu(gate h) * up h)),  h = norm2(x)  (may be missing)

A pass of the loop begins with x <- W [x; x0] + step_t, x0 the scaled
embedding. Each pass has caches and states of its own, so the cache has
entries for every layer run, not per layer.

MI355X layout: the stream is fp32; one launch norms a sublayer's result, adds
it and does the next norm. All inputs of a layer's mixers are one GEMM, and
so are their outputs. W's half for x0 is applied once per step; x enters the
other half as two bf16 terms with an fp32 result, so the stream does not lose
bits to the loop.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Callable, List, Optional, Tuple

import torch
import torch.nn as nn

from helix_amd.engine.weights import Placement
from helix_amd.models.base import (Float32Kept, LayerRun, LoopSpec, round_up,
                                   unroll)
from helix_amd.models.gla import GLASpec
from helix_amd.models.llama import HLinear
from helix_amd.models.mixer_group import GroupSpec, Member, MixerGroup
from helix_amd.models.rotary_attention import (AttnSpec, HalvesRotary,
                                               RotaryTables)
from helix_amd.ops import gated


def sigmoid_mixer(**sizes) -> GroupSpec:
    return GroupSpec((Member(AttnSpec(sigmoid=True, tied_values=True,
                                      bias=True, **sizes)),))


def parallel_mixer(left: dict, left_scale: float, right: GLASpec,
                   right_scale: float) -> GroupSpec:
    return GroupSpec((
        Member(AttnSpec(qk_norm=True, turn_values=True, **left), "left.",
               left_scale),
        Member(right, "right.", right_scale)))


def _attn_sizes(m: dict) -> dict:
    return dict(heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
                vdim=m["vdim"], scale=float(m["scale"]),
                rotary=HalvesRotary.from_json(m.get("rot")))


def _mixer(layer: dict, name: str, rank: Callable[[str], int]) -> GroupSpec:
    m = layer["mixer"]
    if layer["type"] == "attention":
        return sigmoid_mixer(**_attn_sizes(m))
    if layer["type"] == "parallel":
        return parallel_mixer(
            _attn_sizes(m["left"]), float(m["left_scale"]),
            GLASpec.from_json(m["right"], rank(name + ".mix.right.a1")),
            float(m["right_scale"]))
    raise ValueError(f"{name}: unknown mixer {layer['type']!r}")


@dataclass(frozen=True)
class LayerSpec:
    mixer: GroupSpec
    ff: int = 0                  # feed-forward size (0 = none)


@dataclass(frozen=True)
class MotolixConfig:
    name: str
    vocab_size: int
    hidden_size: int
    layers: Tuple[LayerSpec, ...]
    loop: Optional[LoopSpec] = None
    embedding_scale: float = 1.0
    logit_scale: float = 1.0
    norm_eps: float = 1e-5
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
        return [c for r in self.runs()
                for c in self.layers[r.layer].mixer.cache_layers()]

    def num_weights(self) -> Tuple[int, int]:
        """(embedding and head, per-layer total) parameter counts."""
        W = self.hidden_size
        n = sum(l.mixer.num_weights(W) + 3 * W * l.ff for l in self.layers)
        if self.loop is not None:
            n += 2 * W * W
        return 2 * self.vocab_size * W, n

    def activation_bytes(self, tokens: int) -> int:
        """The stream with its loop operands and the widest layer's
        buffers."""
        wide = max(l.mixer.activation_floats() + 2 * l.ff
                   for l in self.layers)
        return tokens * 4 * (7 * self.hidden_size + 2 * wide)

    @classmethod
    def from_json(cls, d: dict, name: str = "motolix",
                  shapes: Optional[dict] = None) -> "MotolixConfig":
        """shapes: checkpoint tensor name -> shape; the rank of a decay's
        projection stands only there."""
        def rank(tensor: str) -> int:
            if not shapes or tensor not in shapes:
                raise ValueError(f"{name}: no tensor {tensor}")
            return int(shapes[tensor][0])

        layers = []
        for i, l in enumerate(d["layers"]):
            mlp = l.get("mlp")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward "
                                 f"{mlp['kind']!r}")
            layers.append(LayerSpec(_mixer(l, f"l{i}", rank),
                                    mlp["ff"] if mlp is not None else 0))
        loop = d.get("loop")
        return cls(
            name=name, vocab_size=d["vocab"], hidden_size=d["width"],
            layers=tuple(layers), loop=None if not loop else LoopSpec(
                loop["start"], loop["stop"], loop["times"]),
            embedding_scale=float((d.get("embedding") or {}).get("scale",
                                                                 1.0)),
            logit_scale=float(d.get("logit_scale", 1.0)),
            norm_eps=float(d["norm"]["eps"]))


def _preset(name, vocab, width, heads, ff, gla_heads, blocks,
            loop) -> MotolixConfig:
    """`blocks` times one sigmoid layer and three parallel ones."""
    D = 128
    rot = HalvesRotary(64, 500000.0, (8.0, 1.0, 4.0, 8192.0))
    one = LayerSpec(sigmoid_mixer(heads=heads, kv_heads=heads // 4, dim=D,
                                  vdim=D, scale=D ** -0.5, rotary=rot), ff)
    two = LayerSpec(parallel_mixer(
        dict(heads=heads // 2, kv_heads=heads // 8, dim=D, vdim=D,
             scale=D ** -0.5, rotary=HalvesRotary(D, 500000.0)), 0.8,
        GLASpec(heads=gla_heads, dim=D, vdim=D, tau=16.0, rank=16), 0.5), ff)
    return MotolixConfig(name=name, vocab_size=vocab, hidden_size=width,
                         layers=(one, two, two, two) * blocks, loop=loop,
                         embedding_scale=width ** 0.5, logit_scale=0.5,
                         max_position=32768)


PRESETS = {
    # 32 layer runs of an 8B-class decoder's sizes over 24 layers
    "motolix-8b": _preset("motolix-8b", 128256, 4096, 32, 14336, 16, 6,
                          LoopSpec(8, 12, 3)),
    "motolix-1b": _preset("motolix-1b", 32000, 2048, 16, 5632, 8, 3,
                          LoopSpec(4, 8, 2)),
    # mixed layers for CPU tests and smoke runs
    "tiny-motolix": MotolixConfig(
        name="tiny-motolix", vocab_size=512, hidden_size=128, layers=(
            LayerSpec(parallel_mixer(
                dict(heads=4, kv_heads=2, dim=24, vdim=40, scale=0.2,
                     rotary=HalvesRotary(16, 1e4)), 0.9,
                GLASpec(heads=3, dim=24, vdim=20, tau=4.0, rank=6), 0.6),
                192),
            LayerSpec(sigmoid_mixer(
                heads=6, kv_heads=2, dim=32, vdim=32, scale=0.2,
                rotary=HalvesRotary(16, 1e5, (2.0, 1.0, 4.0, 128.0))), 0),
            LayerSpec(sigmoid_mixer(
                heads=3, kv_heads=3, dim=16, vdim=16, scale=0.3,
                rotary=HalvesRotary(16, 1e4)), 320),
        ), loop=LoopSpec(0, 2, 2), embedding_scale=11.0, logit_scale=0.7,
        max_position=512),
}


class MotolixLayer(Float32Kept):
    NORMS = ("norm1", "norm1b", "norm2", "norm2b")
    kept = tuple(n + s for n in NORMS for s in ("_w", "_b"))

    def __init__(self, cfg: MotolixConfig, index: int):
        super().__init__()
        spec, W = cfg.layers[index], cfg.hidden_size
        self.spec = spec
        self.mixer = MixerGroup(spec.mixer, W, cfg.norm_eps)
        for n in self.NORMS:
            on = spec.ff or n.startswith("norm1")
            setattr(self, n + "_w",
                    nn.Parameter(torch.ones(W)) if on else None)
            setattr(self, n + "_b",
                    nn.Parameter(torch.zeros(W)) if on else None)
        if spec.ff:
            self.up_at = round_up(spec.ff, 8)
            self.gate_up = HLinear(W, self.up_at + spec.ff, bias=False)
            self.gate_up.weight.data.zero_()
            self.down = HLinear(spec.ff, W, bias=False)

    def norm(self, name: str) -> gated.Norm:
        return gated.Norm(getattr(self, name + "_w"),
                          getattr(self, name + "_b"))

    def feed_forward(self, h):
        return self.down(gated.gated_mul(self.gate_up(h), self.up_at,
                                         self.spec.ff, "gelu_tanh"))

    def targets(self, prefix: str) -> dict:
        out = self.mixer.targets(prefix + "mix.")
        for n in self.NORMS:
            w, b = self.norm(n)
            if w is not None:
                out.update({prefix + n: w.data, prefix + n + ".b": b.data})
        if self.spec.ff:
            w, F = self.gate_up.weight.data, self.spec.ff
            out.update({prefix + "mlp.gate": w[:F],
                        prefix + "mlp.up": w[self.up_at:self.up_at + F],
                        prefix + "mlp.down": self.down.weight.data})
        return out


class MotolixForCausalLM(Float32Kept):
    kept = ("final_w", "final_b", "loop_step")
    paged_prefill = True         # prompts attend through the paged cache
    extension = "_C_gated"       # native library of its kernels

    def __init__(self, cfg: MotolixConfig, tp_size: int = 1,
                 tp_rank: int = 0):
        if tp_size != 1:
            raise ValueError("motolix runs on one GPU: queries and keys are "
                             "normed over all heads (tp_size must be 1)")
        super().__init__()
        self.cfg = cfg
        self.tp_size, self.tp_rank = tp_size, tp_rank
        W = cfg.hidden_size
        self.embed_tokens = nn.Embedding(cfg.vocab_size, W)
        self.layers = nn.ModuleList(
            [MotolixLayer(cfg, i) for i in range(cfg.num_layers)])
        self.loop_x = self.loop_e = self.loop_step = None
        if cfg.loop is not None:
            # the loop's projection, its halves for x and the embedding
            self.loop_x = nn.Parameter(torch.zeros(W, W))
            self.loop_e = nn.Parameter(torch.zeros(W, W))
            self.loop_step = nn.Parameter(torch.zeros(cfg.loop.times, W))
        # the final norm's, times the logits' scale
        self.final_w = nn.Parameter(torch.ones(W))
        self.final_b = nn.Parameter(torch.zeros(W))
        self.lm_head = HLinear(W, cfg.vocab_size, bias=False)
        self.runs = cfg.runs()
        self.cache_at, n = [], 0             # first cache entry of a run
        for r in self.runs:
            self.cache_at.append(n)
            n += len(cfg.layers[r.layer].mixer.members)
        self.cache_at.append(n)
        # optional list receiving the stream after every layer run
        self.layer_tap: Optional[list] = None

    def decode_workspace(self, max_batch: int, max_len: int, device):
        """Flat fp32 scratch, enough for any layer at any batch size."""
        n = max(l.mixer.scratch_floats(max_batch, max_len)
                for l in self.layers)
        return torch.empty(2 * n, dtype=torch.float32, device=device)

    @torch.inference_mode()
    def forward(self, input_ids: torch.Tensor, kv_caches, meta):
        cfg, runs, eps = self.cfg, self.runs, self.cfg.norm_eps
        emb = self.embed_tokens.weight
        dtype = emb.dtype
        tables = RotaryTables(meta.positions)
        x = torch.empty(input_ids.shape[0], cfg.hidden_size,
                        dtype=torch.float32, device=emb.device)
        e = None                             # the embedding's part of a pass
        if cfg.loop is not None:
            e = gated.project32(emb[input_ids], self.loop_e)

        def ahead(run):
            """(norm, operands of the loop's projection) of the row that a
            run starts from; None: the final norm."""
            if run is None:
                return gated.Norm(self.final_w, self.final_b), None
            if run.loop_pass >= 0:
                return None, gated.split_terms(x, dtype)
            return self.layers[run.layer].norm("norm1"), None

        def begin(run, h, terms):
            """A run's input, after its pass has begun."""
            if run is None or run.loop_pass < 0:
                return h
            return gated.stream_enter(
                x, terms, self.loop_x, e, cfg.embedding_scale,
                self.loop_step[run.loop_pass],
                self.layers[run.layer].norm("norm1"), eps, dtype)

        norm, terms = ahead(runs[0])
        h = gated.stream_embed(x, input_ids, emb, cfg.embedding_scale, norm,
                               eps, terms)
        h = begin(runs[0], h, terms)
        for j, run in enumerate(runs):
            layer = self.layers[run.layer]
            nxt = runs[j + 1] if j + 1 < len(runs) else None
            y = layer.mixer(h, kv_caches[self.cache_at[j]:
                                         self.cache_at[j + 1]], meta, tables)
            post = layer.norm("norm1b")
            if layer.spec.ff:
                h = gated.stream_add(x, y, post, layer.norm("norm2"), eps)
                y, post = layer.feed_forward(h), layer.norm("norm2b")
            tap = None
            if self.layer_tap is not None:
                tap = torch.empty_like(x)
                self.layer_tap.append(tap)
            norm, terms = ahead(nxt)
            h = gated.stream_add(x, y, post, norm, eps, terms, tap)
            h = begin(nxt, h, terms)
        return h

    @torch.inference_mode()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return self.lm_head(hidden)

    # ------------------------------------------------------------------
    def checkpoint_targets(self) -> dict:
        """Checkpoint tensor name -> the view or Placement it is loaded
        into."""
        W, s = self.cfg.hidden_size, self.cfg.logit_scale
        out = {"embed": self.embed_tokens.weight.data,
               "head": self.lm_head.weight.data,
               "final.norm": Placement((W,), [
                   (self.final_w.data, lambda t: t.float() * s)]),
               "final.norm.b": Placement((W,), [
                   (self.final_b.data, lambda t: t.float() * s)])}
        if self.loop_step is not None:
            out["loop.in"] = Placement((W, 2 * W), [
                (self.loop_x.data, lambda t: t[:, :W]),
                (self.loop_e.data, lambda t: t[:, W:])])
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
            if leaf in ("norm", "temp") or leaf in MotolixLayer.NORMS:
                fill(t, 0.05, 1.0)
            elif name.endswith("a2.b"):
                fill(t, 1.0, 2.0)
            elif leaf == "pb":
                fill(t, 0.5, -2.0)
            elif name == "loop.in":
                fill(t, (2.0 * self.cfg.hidden_size) ** -0.5)
            else:
                fill(t, 0.02)
        return self

    def memory_bytes(self) -> int:
        return sum(p.numel() * p.element_size() for p in self.parameters())
