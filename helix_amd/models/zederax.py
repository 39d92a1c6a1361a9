"""Zederax: parallel attention / feed-forward layers over a depth-averaged
fp32 residual stream.

Per layer i, with h = RMSNorm(x):

    X_{i+1} = x + attention(h) + feed_forward(h)
    x       = sum_{j <= i+1} dwa_i[j] X_j          (X_0 = embedding)

attention: unit-RMS q and k heads, soft-capped scores minus a per-head
distance bias, sliding window, softmax, talking heads (the softmaxed
weights are mixed across heads), values blended with those of the first
value-mixing layer, one sigmoid gate per head. feed_forward: up -> PolyNorm
-> down. The output head is the embedding table.

MI355X layout: both sublayers read the same h, so a layer is two GEMMs: one
for [q | k | v | up | gate] and one for [o | down], whose fp32 accumulator
adds the two sublayers. Around them run one epilogue launch (unit norms,
value mixing, cache write, PolyNorm), the paged talking-head attention, and
one launch for residual add + depth average + the next layer's norm.
"""
from __future__ import annotations

from dataclasses import dataclass, replace
from typing import List, Optional, Tuple

import torch
import torch.nn as nn

from helix_amd import ops
from helix_amd.models.base import Float32Kept, round_up
from helix_amd.models.llama import HLinear
from helix_amd.models.meta import KVLayer, MixedMeta


@dataclass(frozen=True)
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int                     # query / key head size
    vdim: int                    # value head size
    window: int                  # visible tokens, own included (0 = all)
    scale: float
    softcap: float = 0.0         # 0 = none
    v_mix: bool = False

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads over {self.kv_heads} "
                             "key/value heads")


@dataclass(frozen=True)
class LayerSpec:
    mixer: AttentionSpec
    ff: int = 0                  # feed-forward size (0 = none)


@dataclass(frozen=True)
class ZederaxConfig:
    name: str
    vocab_size: int
    hidden_size: int
    layers: Tuple[LayerSpec, ...]
    rms_norm_eps: float = 1e-6
    max_position: int = 1 << 20  # nothing in the design bounds it

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def kv_layers(self, tp_size: int = 1) -> List[KVLayer]:
        return [KVLayer(l.mixer.kv_heads, round_up(l.mixer.dim, 8), l.mixer.vdim,
                        v_transposed=True) for l in self.layers]

    def num_weights(self) -> Tuple[int, int]:
        """(embedding, per-layer total) parameter counts."""
        n = 0
        for l in self.layers:
            m = l.mixer
            n += self.hidden_size * (
                m.heads * (m.dim + m.vdim + 1)
                + m.kv_heads * (m.dim + m.vdim) + 2 * l.ff)
        return self.vocab_size * self.hidden_size, n

    def activation_bytes(self, tokens: int) -> int:
        """Depth history plus the widest layer's buffers."""
        wide = max(l.mixer.heads * (2 * l.mixer.dim + 2 * l.mixer.vdim)
                   + 2 * l.ff for l in self.layers)
        return tokens * (4 * self.hidden_size * (self.num_layers + 2)
                         + 4 * wide)

    @classmethod
    def from_json(cls, d: dict, name: str = "zederax") -> "ZederaxConfig":
        layers = []
        for i, l in enumerate(d["layers"]):
            if l["type"] != "attention":
                raise ValueError(f"layer {i}: unknown mixer {l['type']!r}")
            m, mlp = l["mixer"], l.get("mlp")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward "
                                 f"{mlp['kind']!r}")
            layers.append(LayerSpec(
                AttentionSpec(
                    heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
                    vdim=m["vdim"],
                    window=int((m.get("mask") or {}).get("size") or 0),
                    scale=float(m["scale"]),
                    softcap=float(m.get("softcap") or 0.0),
                    v_mix=bool(m.get("v_mix", False))),
                ff=mlp["ff"] if mlp is not None else 0))
        return cls(name=name, vocab_size=d["vocab"], hidden_size=d["width"],
                   layers=tuple(layers),
                   rms_norm_eps=float(d["norm"]["eps"]))


def _uniform(name, vocab, width, depth, ff, attn: AttentionSpec,
             max_position) -> ZederaxConfig:
    return ZederaxConfig(name=name, vocab_size=vocab, hidden_size=width,
                         layers=(LayerSpec(attn, ff),) * depth,
                         max_position=max_position)


PRESETS = {
    # the layer sizes of an 8B-class GQA decoder; the feed-forward has two
    # matrices instead of three, so ff is 1.5x
    "zederax-8b": _uniform(
        "zederax-8b", 128256, 4096, 32, 21504,
        AttentionSpec(heads=32, kv_heads=8, dim=128, vdim=128, window=4096,
                      scale=128 ** -0.5, softcap=50.0, v_mix=True), 8192),
    "zederax-1b": _uniform(
        "zederax-1b", 32000, 2048, 16, 8448,
        AttentionSpec(heads=16, kv_heads=4, dim=128, vdim=128, window=2048,
                      scale=128 ** -0.5, softcap=50.0, v_mix=True), 8192),
    # mixed layers for CPU tests and smoke runs
    "tiny-zederax": ZederaxConfig(
        name="tiny-zederax", vocab_size=512, hidden_size=128, layers=(
            LayerSpec(AttentionSpec(6, 2, 40, 24, 24, 0.2, 30.0, True), 192),
            LayerSpec(AttentionSpec(3, 3, 16, 64, 40, 0.3, 20.0, False), 0),
            LayerSpec(AttentionSpec(6, 2, 32, 24, 17, 0.25, 0.0, True), 320),
        ), rms_norm_eps=1e-5, max_position=512),
}


class ZederaxLayer(Float32Kept):
    kept = ("norm_w", "talk", "vmix", "act", "dwa", "slopes")

    def __init__(self, cfg: ZederaxConfig, index: int):
        super().__init__()
        spec = cfg.layers[index]
        m = spec.mixer
        self.spec, self.m = spec, m
        W, H, G = cfg.hidden_size, m.heads, m.kv_heads
        # column starts in the fused projection, 16-byte aligned
        self.cols, at = {}, 0
        for name, n in (("q", H * m.dim), ("k", G * m.dim),
                        ("v", G * m.vdim), ("up", spec.ff), ("g", H)):
            self.cols[name] = (at, n)
            at = round_up(at + n, 8)
        self.in_proj = HLinear(W, round_up(at, 64), bias=True)
        # [o | down] share the accumulator
        self.down_at = round_up(H * m.vdim, 8)
        self.out_width = round_up(self.down_at + spec.ff, 8)
        self.out_proj = HLinear(self.out_width, W, bias=False)
        for p in (self.in_proj.weight, self.in_proj.bias,
                  self.out_proj.weight):
            p.data.zero_()
        self.norm_w = nn.Parameter(torch.ones(W))
        self.talk = nn.Parameter(torch.eye(H))
        self.vmix = nn.Parameter(torch.zeros(())) if m.v_mix else None
        self.act = nn.Parameter(torch.tensor([1.0, 0.0, 0.0, 0.0])) \
            if spec.ff else None
        dwa = torch.zeros(index + 2)
        dwa[-1] = 1.0
        self.dwa = nn.Parameter(dwa)
        self.register_buffer("slopes", torch.tensor(
            [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)],
            dtype=torch.float64).float(), persistent=False)

    @property
    def talk_params(self) -> ops.TalkParams:
        m = self.m
        return ops.TalkParams(m.scale, m.softcap, m.window, self.slopes,
                              self.talk)

    def _cols(self, z: torch.Tensor, name: str) -> torch.Tensor:
        at, n = self.cols[name]
        return z[:, at:at + n]

    def forward(self, h, kv_cache, meta, v_first, first: bool, buf, eps):
        """Both sublayers' sum for the rows h. v_first: the value-mixing
        carry (written by the first such layer). buf: [T, out_width]."""
        m, spec = self.m, self.spec
        z = self.in_proj(h)
        ff = None
        if spec.ff:
            ff = (self._cols(z, "up"),
                  buf[:, self.down_at:self.down_at + spec.ff], self.act)
        q = ops.unit_qkv_cache(
            z, [self.cols[n][0] for n in ("q", "k", "v")], m.heads, m.dim,
            kv_cache, meta.slot_mapping, eps,
            v_first=v_first if m.v_mix else None,
            lam=self.vmix if m.v_mix else None, first=first, ff=ff)
        self.attend(buf[:, :m.heads * m.vdim], q, kv_cache, meta,
                    self._cols(z, "g"))
        return self.out_proj(buf)

    def attend(self, out, q, kv_cache, meta, gate):
        p = self.talk_params
        if isinstance(meta, MixedMeta):
            n = meta.num_decode
            self._attend_rows(out[:n], q[:n], kv_cache, meta.decode, gate[:n],
                              p)
            self._attend_prompt(out[n:], q[n:], kv_cache, meta.prefill,
                                gate[n:], p)
        elif meta.is_prefill:
            self._attend_prompt(out, q, kv_cache, meta, gate, p)
        else:
            self._attend_rows(out, q, kv_cache, meta, gate, p)

    @staticmethod
    def _attend_rows(out, q, kv_cache, meta, gate, p):
        ops.talk_attn_rows(out, q, kv_cache, meta.block_tables,
                           meta.seq_lens, meta.max_len, p, gate,
                           workspace=meta.workspace)

    @staticmethod
    def _attend_prompt(out, q, kv_cache, meta, gate, p):
        ops.talk_attn_prefill(out, q, kv_cache, meta.block_tables,
                              meta.cu_seqlens, meta.seq_lens,
                              meta.max_seqlen, meta.max_len, meta.row_seq,
                              meta.row_len, p, gate)


class ZederaxForCausalLM(Float32Kept):
    kept = ("final_norm_w",)
    paged_prefill = True         # prompts attend through the paged cache
    extension = "_C_ext"         # native library of its kernels

    def __init__(self, cfg: ZederaxConfig, tp_size: int = 1,
                 tp_rank: int = 0):
        if tp_size != 1:
            raise ValueError("zederax runs on one GPU: talking heads mix "
                             "all heads of a token (tp_size must be 1)")
        super().__init__()
        self.cfg = cfg
        self.tp_size, self.tp_rank = tp_size, tp_rank
        self.embed_tokens = nn.Embedding(cfg.vocab_size, cfg.hidden_size)
        self.layers = nn.ModuleList(
            [ZederaxLayer(cfg, i) for i in range(cfg.num_layers)])
        self.final_norm_w = nn.Parameter(torch.ones(cfg.hidden_size))
        mixing = [i for i, l in enumerate(cfg.layers) if l.mixer.v_mix]
        self.first_v_mix = mixing[0] if mixing else -1
        shapes = {(cfg.layers[i].mixer.kv_heads, cfg.layers[i].mixer.vdim)
                  for i in mixing}
        if len(shapes) > 1:
            raise ValueError("value mixing needs equally shaped values in "
                             f"all its layers, got {sorted(shapes)}")
        # optional list receiving the stream after every layer
        self.layer_tap: Optional[list] = None

    def decode_workspace(self, max_batch: int, max_len: int, device):
        """Flat fp32 scratch, enough for any layer at any batch size."""
        n = 0
        for l in self.cfg.layers:
            m = l.mixer
            keys = min(max_len, m.window) if m.window else max_len
            for rows in {1, max_batch} | {
                    b for b in (2 ** i for i in range(12)) if b < max_batch}:
                n = max(n, ops.talk_scratch_floats(
                    rows, m.heads, m.kv_heads, m.vdim, keys))
        return torch.empty(2 * n, dtype=torch.float32, device=device)

    @torch.inference_mode()
    def forward(self, input_ids: torch.Tensor, kv_caches, meta):
        cfg = self.cfg
        T, L, eps = input_ids.shape[0], cfg.num_layers, cfg.rms_norm_eps
        emb = self.embed_tokens.weight
        dev, dtype = emb.device, emb.dtype
        hist = torch.empty(L, T, cfg.hidden_size, dtype=torch.float32,
                           device=dev)
        x = hist[0]
        x_avg = torch.empty_like(x)
        h = ops.embed_norm(input_ids, emb, self.layers[0].norm_w, eps, x)
        v_first = None
        if self.first_v_mix >= 0:
            m = cfg.layers[self.first_v_mix].mixer
            v_first = torch.empty(T, m.kv_heads * m.vdim, dtype=dtype,
                                  device=dev)
        bufs = {}
        for i, layer in enumerate(self.layers):
            key = (layer.m.heads * layer.m.vdim, layer.spec.ff)
            if key not in bufs:
                bufs[key] = torch.empty(T, layer.out_width, dtype=dtype,
                                        device=dev)
                for a, b in ((key[0], layer.down_at),
                             (layer.down_at + key[1], layer.out_width)):
                    if b > a:
                        bufs[key][:, a:b].zero_()
            y = layer(h, kv_caches[i], meta, v_first, i == self.first_v_mix,
                      bufs[key], eps)
            last = i == L - 1
            keep_x = not last or self.layer_tap is not None
            h = ops.depth_norm(
                x, y, hist, i + 1, layer.dwa,
                self.final_norm_w if last else self.layers[i + 1].norm_w,
                eps, store_new=not last, x_out=x_avg if keep_x else None)
            x = x_avg
            if self.layer_tap is not None:
                self.layer_tap.append(x.clone())
        return h

    @torch.inference_mode()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return ops.linear(hidden, self.embed_tokens.weight)

    # ------------------------------------------------------------------
    def checkpoint_targets(self) -> dict:
        """Checkpoint tensor name -> the view it is loaded into."""
        out = {"embed": self.embed_tokens.weight.data,
               "final.norm": self.final_norm_w.data}
        for i, l in enumerate(self.layers):
            w, b, o = (l.in_proj.weight.data, l.in_proj.bias.data,
                       l.out_proj.weight.data)

            def rows(name, t, l=l):
                at, n = l.cols[name]
                return t[at:at + n]

            p = f"l{i}."
            out[p + "norm1"] = l.norm_w.data
            out[p + "dwa"] = l.dwa.data
            for n in ("q", "k", "v"):
                out[f"{p}mix.{n}"] = rows(n, w)
                out[f"{p}mix.{n}.b"] = rows(n, b)
            out[p + "mix.g"] = rows("g", w)
            out[p + "mix.talk"] = l.talk.data
            if l.vmix is not None:
                out[p + "mix.vmix"] = l.vmix.data
            out[p + "mix.o"] = o[:, :l.m.heads * l.m.vdim]
            if l.spec.ff:
                out[p + "mlp.up"] = rows("up", w)
                out[p + "mlp.act"] = l.act.data
                out[p + "mlp.down"] = o[:, l.down_at:l.down_at + l.spec.ff]
        return out

    def optional_checkpoint_names(self) -> set:
        """The first value-mixing layer never uses its coefficient."""
        return {f"l{self.first_v_mix}.mix.vmix"}

    @torch.inference_mode()
    def init_random(self, seed: int = 0):
        """Random weights with every mechanism active."""
        dev = self.embed_tokens.weight.device
        g = torch.Generator(device=dev).manual_seed(seed)

        def normal(t, std, mean=0.0):
            t.copy_(torch.randn(t.shape, generator=g, device=dev) * std
                    + mean)

        for name, t in self.checkpoint_targets().items():
            leaf = name.rsplit(".", 1)[-1]
            if name.endswith("norm") or leaf == "norm1":
                normal(t, 0.05, 1.0)
            elif leaf == "talk":
                t.copy_(torch.eye(t.shape[0], device=dev)
                        + 0.1 * torch.randn(t.shape, generator=g, device=dev))
            elif leaf == "vmix":
                t.fill_(0.3)
            elif leaf == "act":
                t.copy_(torch.tensor([0.8, 0.3, 0.2, 0.05], device=dev))
            elif leaf == "dwa":
                normal(t, 0.05)
                t[-1] += 1.0
            else:
                normal(t, 0.02)
        return self

    def memory_bytes(self) -> int:
        return sum(p.numel() * p.element_size() for p in self.parameters())


def with_window(cfg: ZederaxConfig, window: int) -> ZederaxConfig:
    """The same model with another window in every layer."""
    return replace(cfg, layers=tuple(
        replace(l, mixer=replace(l.mixer, window=window))
        for l in cfg.layers))
