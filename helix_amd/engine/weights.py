"""Weight IO: safetensors load/save with HF-checkpoint name mapping and
pinned-host + side-stream async H2D staging (SURVEY.md §2.8 "Weight
load": replaces vLLM's HF download/load with a native path that does not
stall serving streams).
"""
from __future__ import annotations

import glob
import json
import logging
import os
from dataclasses import dataclass
from typing import Callable, Dict, Iterator, List, Tuple

import torch

log = logging.getLogger("helix_amd.weights")


def save_sharded(model: torch.nn.Module, out_dir: str,
                 shard_bytes: int = 4 << 30):
    """Save a model as safetensors shards (our native checkpoint format)."""
    from safetensors.torch import save_file
    os.makedirs(out_dir, exist_ok=True)
    shard: Dict[str, torch.Tensor] = {}
    size = 0
    idx = 0
    index = {}
    sd = model.state_dict()
    for name, t in sd.items():
        tb = t.detach().cpu().contiguous()
        shard[name] = tb
        size += tb.numel() * tb.element_size()
        if size >= shard_bytes:
            fn = f"model-{idx:05d}.safetensors"
            save_file(shard, os.path.join(out_dir, fn))
            for n in shard:
                index[n] = fn
            shard, size = {}, 0
            idx += 1
    if shard:
        fn = f"model-{idx:05d}.safetensors"
        save_file(shard, os.path.join(out_dir, fn))
        for n in shard:
            index[n] = fn
    with open(os.path.join(out_dir, "model.safetensors.index.json"),
              "w") as f:
        json.dump({"weight_map": index}, f)


def iter_safetensors(ckpt_dir: str) -> Iterator[Tuple[str, torch.Tensor]]:
    from safetensors import safe_open
    files = sorted(glob.glob(os.path.join(ckpt_dir, "*.safetensors")))
    if not files:
        raise FileNotFoundError(f"no .safetensors under {ckpt_dir}")
    for path in files:
        with safe_open(path, framework="pt", device="cpu") as f:
            for name in f.keys():
                yield name, f.get_tensor(name)


def tensor_shapes(ckpt_dir: str) -> Dict[str, Tuple[int, ...]]:
    """Shape of every tensor of a checkpoint folder."""
    from safetensors import safe_open
    out = {}
    for path in sorted(glob.glob(os.path.join(ckpt_dir, "*.safetensors"))):
        with safe_open(path, framework="pt", device="cpu") as f:
            for name in f.keys():
                out[name] = tuple(f.get_slice(name).get_shape())
    return out


# HF Llama checkpoint name -> (our param, role). Roles q/k/v and
# gate/up are packed into the fused projections.
def _map_hf_name(name: str):
    name = name.replace("model.", "")
    if name == "embed_tokens.weight":
        return "embed_tokens.weight", None
    if name == "norm.weight":
        return "final_norm_w", None
    if name == "lm_head.weight":
        return "lm_head.weight", None
    if name.startswith("layers."):
        parts = name.split(".")
        i = parts[1]
        rest = ".".join(parts[2:])
        m = {
            "input_layernorm.weight": (f"layers.{i}.input_norm_w", None),
            "post_attention_layernorm.weight":
                (f"layers.{i}.post_norm_w", None),
            "self_attn.q_proj.weight":
                (f"layers.{i}.attn.qkv_proj.weight", "q"),
            "self_attn.k_proj.weight":
                (f"layers.{i}.attn.qkv_proj.weight", "k"),
            "self_attn.v_proj.weight":
                (f"layers.{i}.attn.qkv_proj.weight", "v"),
            "self_attn.q_proj.bias":
                (f"layers.{i}.attn.qkv_proj.bias", "q"),
            "self_attn.k_proj.bias":
                (f"layers.{i}.attn.qkv_proj.bias", "k"),
            "self_attn.v_proj.bias":
                (f"layers.{i}.attn.qkv_proj.bias", "v"),
            "self_attn.o_proj.weight":
                (f"layers.{i}.attn.o_proj.weight", None),
            "mlp.gate_proj.weight":
                (f"layers.{i}.mlp.gate_up_proj.weight", "gate"),
            "mlp.up_proj.weight":
                (f"layers.{i}.mlp.gate_up_proj.weight", "up"),
            "mlp.down_proj.weight":
                (f"layers.{i}.mlp.down_proj.weight", None),
        }
        if rest in m:
            return m[rest]
    return name, None  # our native names pass through


class _Stager:
    """Copies host tensors to their destination views. On GPU they go
    through double-buffered pinned memory and a side stream; a buffer's
    event is waited for before the buffer is refilled."""

    def __init__(self, device, use_async: bool = True):
        self.device = device
        self.side = torch.cuda.Stream(device) \
            if (device.type == "cuda" and use_async) else None
        self.pinned = [None, None]
        self.events = [None, None]
        self.cur = 0

    def copy(self, dst_view: torch.Tensor, src: torch.Tensor):
        src = src.to(dst_view.dtype)
        if self.side is None:
            dst_view.copy_(src)
            return
        cur = self.cur
        n = src.numel() * src.element_size()
        if self.pinned[cur] is None or self.pinned[cur].numel() < n:
            self.pinned[cur] = torch.empty(max(n, 64 << 20),
                                           dtype=torch.uint8, pin_memory=True)
            self.events[cur] = torch.cuda.Event()
        else:
            self.events[cur].synchronize()
        flat = self.pinned[cur][:n]
        flat.copy_(src.contiguous().view(-1).view(torch.uint8))
        with torch.cuda.stream(self.side):
            if dst_view.is_contiguous():
                dst_view.view(-1).view(torch.uint8).copy_(flat,
                                                          non_blocking=True)
            else:
                dst_view.copy_(flat.view(src.dtype).view(src.shape),
                               non_blocking=True)
            self.events[cur].record(self.side)
        self.cur ^= 1

    def finish(self):
        if self.side is not None:
            torch.cuda.current_stream(self.device).wait_stream(self.side)
            torch.cuda.synchronize(self.device)


@torch.inference_mode()
def load_llama_weights(model, ckpt_dir: str, use_async: bool = True):
    """Load a Llama checkpoint (HF layout or our native layout) into the
    model. On GPU, tensors are staged through a pinned-host buffer and
    copied on a side stream (hipMemcpyAsync) so decode streams on the
    default stream are not serialized behind weight traffic."""
    # GGUF checkpoints (llama.cpp ecosystem) route through the native
    # GGUF loader (engine/gguf.py): file path or a dir holding one.
    gguf_path = None
    if ckpt_dir.endswith(".gguf") and os.path.isfile(ckpt_dir):
        gguf_path = ckpt_dir
    elif os.path.isdir(ckpt_dir):
        ggufs = sorted(glob.glob(os.path.join(ckpt_dir, "*.gguf")))
        if ggufs and not glob.glob(os.path.join(ckpt_dir, "*.safetensors")):
            gguf_path = ggufs[0]
    if gguf_path is not None:
        from . import gguf as _gguf
        n = _gguf.load_gguf_weights(model, gguf_path)
        log.info("loaded %d tensors from GGUF %s", n, gguf_path)
        return n

    params = dict(model.named_parameters())
    cfg = model.cfg
    q, kv = cfg.q_size, cfg.kv_size
    inter = cfg.intermediate_size
    stager = _Stager(next(model.parameters()).device, use_async)
    stage_copy = stager.copy

    loaded = 0
    for name, tensor in iter_safetensors(ckpt_dir):
        our, role = _map_hf_name(name)
        if our not in params:
            log.debug("skipping unknown weight %s", name)
            continue
        p = params[our]
        if role == "q":
            stage_copy(p.data[:q], tensor)
        elif role == "k":
            stage_copy(p.data[q:q + kv], tensor)
        elif role == "v":
            stage_copy(p.data[q + kv:], tensor)
        elif role == "gate":
            stage_copy(p.data[:inter], tensor)
        elif role == "up":
            stage_copy(p.data[inter:], tensor)
        else:
            stage_copy(p.data, tensor)
        loaded += 1
    stager.finish()
    log.info("loaded %d tensors from %s", loaded, ckpt_dir)
    return loaded


@dataclass
class Placement:
    """Where a checkpoint tensor goes when that is not one view of its own
    shape: into padded rows, or into several layouts. parts: (destination,
    function of the stored tensor)."""
    shape: Tuple[int, ...]
    parts: List[Tuple[torch.Tensor, Callable]]

    @property
    def device(self):
        return self.parts[0][0].device

    def copy_(self, src: torch.Tensor, copy: Callable = torch.Tensor.copy_):
        for dst, fn in self.parts:
            copy(dst, fn(src))


@torch.inference_mode()
def load_mapped_weights(model, ckpt_dir: str, use_async: bool = True) -> int:
    """Load a checkpoint through the model's own name map
    (checkpoint_targets: tensor name -> destination view or Placement).
    Every target has to be there, with its exact shape."""
    targets = model.checkpoint_targets()
    missing = set(targets) - set(model.optional_checkpoint_names())
    stager = _Stager(next(model.parameters()).device, use_async)
    loaded = 0
    for name, tensor in iter_safetensors(ckpt_dir):
        dst = targets.get(name)
        if dst is None:
            log.debug("skipping unknown weight %s", name)
            continue
        if tuple(tensor.shape) != tuple(dst.shape):
            raise ValueError(f"{name}: checkpoint has {tuple(tensor.shape)}, "
                             f"the configuration {tuple(dst.shape)}")
        if isinstance(dst, Placement):
            dst.copy_(tensor, stager.copy)
        else:
            stager.copy(dst, tensor)
        missing.discard(name)
        loaded += 1
    stager.finish()
    if missing:
        raise ValueError(f"{ckpt_dir} lacks {sorted(missing)}")
    log.info("loaded %d tensors from %s", loaded, ckpt_dir)
    return loaded


def load_weights(model, ckpt_dir: str, use_async: bool = True) -> int:
    """Load a checkpoint into any causal LM of the registry."""
    if hasattr(model, "checkpoint_targets"):
        return load_mapped_weights(model, ckpt_dir, use_async)
    return load_llama_weights(model, ckpt_dir, use_async)
