"""Model registry: a preset name or a checkpoint folder -> configuration,
model class and weight loader.

A folder is recognised by its config.json ("architecture", or the
"architectures" list of the Hugging Face layout).
"""
from __future__ import annotations

import json
import os
from typing import Callable, Dict, Optional

from helix_amd.models import dibizen, llama, motolix, nibezen, zederax
from helix_amd.models.dibizen import DibizenConfig, DibizenForCausalLM
from helix_amd.models.llama import LlamaConfig, LlamaForCausalLM
from helix_amd.models.motolix import MotolixConfig, MotolixForCausalLM
from helix_amd.models.nibezen import NibezenConfig, NibezenForCausalLM
from helix_amd.models.zederax import ZederaxConfig, ZederaxForCausalLM

MODEL_CLASSES = {DibizenConfig: DibizenForCausalLM,
                 LlamaConfig: LlamaForCausalLM,
                 MotolixConfig: MotolixForCausalLM,
                 NibezenConfig: NibezenForCausalLM,
                 ZederaxConfig: ZederaxForCausalLM}

# config.json architecture -> reader(dict, name) of the configuration
CONFIG_READERS: Dict[str, Callable] = {
    "Dibizen": DibizenConfig.from_json,
    "Motolix": MotolixConfig.from_json,
    "Nibezen": NibezenConfig.from_json,
    "Zederax": ZederaxConfig.from_json,
    "LlamaForCausalLM": LlamaConfig.from_json,
    "MistralForCausalLM": LlamaConfig.from_json,
    "Qwen2ForCausalLM": LlamaConfig.from_json,
}

# designs whose config.json leaves some sizes to the tensors' shapes
SIZED_BY_TENSORS = {"Motolix"}


def is_folder(model: str) -> bool:
    return os.path.isfile(os.path.join(model, "config.json"))


def get_config(model: str):
    """Configuration of a preset or of a checkpoint folder."""
    families = (dibizen.PRESETS, llama.PRESETS, motolix.PRESETS,
                nibezen.PRESETS, zederax.PRESETS)
    for presets in families:
        if model in presets:
            return presets[model]
    if not is_folder(model):
        known = sorted(name for presets in families for name in presets)
        raise KeyError(f"unknown model {model!r}: neither a folder with "
                       f"config.json nor one of {known}")
    with open(os.path.join(model, "config.json")) as f:
        d = json.load(f)
    arch = d.get("architecture") or (d.get("architectures") or [None])[0]
    if arch not in CONFIG_READERS:
        raise ValueError(f"{model}: unknown architecture {arch!r}")
    name = os.path.basename(os.path.normpath(model))
    sizes = {}
    if arch in SIZED_BY_TENSORS:
        from helix_amd.engine import weights
        sizes["shapes"] = weights.tensor_shapes(model)
    return CONFIG_READERS[arch](d, name=name, **sizes)


def model_class(cfg):
    return MODEL_CLASSES[type(cfg)]


def build_model(model: str, dtype, device, seed: int = 0, tp_size: int = 1,
                tp_rank: int = 0, cfg: Optional[object] = None):
    """Instantiate on `device`; weights come from the folder, or are random
    for a preset."""
    from helix_amd.engine import weights
    cfg = cfg if cfg is not None else get_config(model)
    m = model_class(cfg)(cfg, tp_size, tp_rank)
    m = m.to(dtype).to(device)
    if is_folder(model):
        if tp_size != 1:
            raise ValueError("checkpoint folders load on one GPU")
        weights.load_weights(m, model)
    else:
        m.init_random(seed)
    return m
