# SPDX-License-Identifier: Apache-2.0
"""Model registry: which architectures are served, and how a checkpoint's config.json becomes a configuration object.

A layer-stack design registers a reader of its config.json; the object it returns carries the attributes the worker
reads off a HuggingFace config and a `stack` dictionary, the library's description of the model (mi_stack_config in
include/mi355x_vllm.h).  Llama-family checkpoints keep their HuggingFace config and have no `stack`."""

from __future__ import annotations

import json
import os
from types import SimpleNamespace

from .._stack_enums import MI_MIX
from .bokulorn import BokulornConfig
from .nusovik import NusovikConfig
from .rapodra import RapodraConfig
from .vimesun import VimesunConfig

# served through multimodal model classes by the reference: out of this backend's scope
MULTI_MODAL_MODELS = [f"{family}ForConditionalGeneration" for family in ("Mllama", "Llava", "Llama4")]

LLAMA_FAMILY = ("LlamaForCausalLM", "Qwen2ForCausalLM", "MistralForCausalLM")
# architecture name -> reader of its config.json dictionary
STACK_DESIGNS = {design.architecture: design.from_dict for design in (VimesunConfig, RapodraConfig, BokulornConfig, NusovikConfig)}
SUPPORTED_ARCHITECTURES = LLAMA_FAMILY + tuple(STACK_DESIGNS)


def config_from_dict(raw: dict):
    """config.json contents -> configuration object."""
    arch = raw.get("architecture") or (raw.get("architectures") or [None])[0]
    if arch in STACK_DESIGNS:
        return STACK_DESIGNS[arch](raw)
    if arch is None:
        raise ValueError("config.json names no architecture")
    if arch not in SUPPORTED_ARCHITECTURES:
        raise ValueError(f"Model {arch} is not supported on MI355X for now. "
                         f"Supported models: {list(SUPPORTED_ARCHITECTURES)}")
    return SimpleNamespace(**raw)


def load_config(model_dir: str):
    with open(os.path.join(model_dir, "config.json"), "r", encoding="utf-8") as f:
        return config_from_dict(json.load(f))


def stack_of(config) -> dict | None:
    """The library's description of a layer-stack model; None for the Llama family."""
    return getattr(config, "stack", None)


def has_recurrent_state(config) -> bool:
    """Whether a sequence owns state that is not in KV blocks (a slot per sequence; no prefix to be taken over from the cache)."""
    stack = stack_of(config)
    recurrent = {MI_MIX["delta"], MI_MIX["scan"], MI_MIX["ssd"]}
    return stack is not None and any(x.get(k) in recurrent for x in stack["layers"] for k in ("mixer_kind", "beside_kind"))


def fill_sizes(config, shape_of) -> None:
    """Sizes a design's config.json leaves to the checkpoint: `shape_of`(tensor name) -> its shape, or None."""
    for (layer, name), tensor in getattr(config, "sizes_from", {}).items():
        if config.stack["layers"][layer].get(name):
            continue
        shape = shape_of(tensor)
        if shape is None:
            raise ValueError(f"{config.architecture}: tensor {tensor}, whose shape gives {name} of layer {layer}, is not in the checkpoint")
        config.stack["layers"][layer][name] = int(shape[0])
