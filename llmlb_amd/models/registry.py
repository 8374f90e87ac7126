"""Model registry: architectures, presets and model folders.

A model is named by a preset ("llama-3-8b") or by a folder that holds
config.json and *.safetensors; config.json's "architecture" picks the
class.
"""
from __future__ import annotations

import json
from pathlib import Path

from .dibelix import DibelixConfig, DibelixForCausalLM
from .fidepel import FidepelConfig, FidepelForCausalLM
from .llama import LlamaConfig, LlamaForCausalLM
from .rasodra import RasodraConfig, RasodraForCausalLM
from .taletar import TaletarConfig, TaletarForCausalLM

MODELS = {
    LlamaConfig: LlamaForCausalLM,
    DibelixConfig: DibelixForCausalLM,
    TaletarConfig: TaletarForCausalLM,
    FidepelConfig: FidepelForCausalLM,
    RasodraConfig: RasodraForCausalLM,
}

# architectures that can be read from a model folder
FOLDERS = {
    DibelixConfig.architecture: DibelixConfig,
    TaletarConfig.architecture: TaletarConfig,
    FidepelConfig.architecture: FidepelConfig,
    RasodraConfig.architecture: RasodraConfig,
}

PRESETS = {
    "llama-3-8b": LlamaConfig.llama3_8b,
    "llama-3-70b": LlamaConfig.llama3_70b,
    "qwen2-7b": LlamaConfig.qwen2_7b,
    "qwen2-0.5b": LlamaConfig.qwen2_0_5b,
    "llama-tiny": LlamaConfig.tiny,
    "llama-small": LlamaConfig.small,
    "dibelix-tiny": DibelixConfig.tiny,
    "dibelix-small": DibelixConfig.small,
    "dibelix-8b": DibelixConfig.base_8b,
    "taletar-tiny": TaletarConfig.tiny,
    "taletar-small": TaletarConfig.small,
    "taletar-8b": TaletarConfig.base_8b,
    "fidepel-tiny": FidepelConfig.tiny,
    "fidepel-small": FidepelConfig.small,
    "fidepel-8b": FidepelConfig.base_8b,
    "rasodra-tiny": RasodraConfig.tiny,
    "rasodra-small": RasodraConfig.small,
    "rasodra-8b": RasodraConfig.base_8b,
}


def resolve(model: str):
    """(config, folder with its weights or None) of a preset or a model
    folder."""
    if model in PRESETS:
        return PRESETS[model](), None
    folder = Path(model)
    if not (folder / "config.json").is_file():
        raise SystemExit(f"unknown model preset '{model}' and no folder "
                         f"with a config.json (presets: "
                         f"{', '.join(PRESETS)})")
    arch = json.loads((folder / "config.json").read_text()).get(
        "architecture")
    if arch not in FOLDERS:
        raise SystemExit(f"unknown architecture '{arch}' in {folder} "
                         f"(have: {', '.join(FOLDERS)})")
    return FOLDERS[arch].from_dir(folder), str(folder)


def model_class(cfg):
    return MODELS[type(cfg)]
