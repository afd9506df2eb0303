"""Which class loads a model: a GGUF file is the quantised Llama family (model.py), a folder with config.json and
model.safetensors is a layer-stack design chosen by the configuration's "architecture" (designs/)."""
from __future__ import annotations

import json
import os

from . import _lib
from .model import HipModel


def architectures():
    from .designs import DESIGNS
    return ["llama (GGUF)"] + sorted(DESIGNS)


def is_model_folder(path: str) -> bool:
    return os.path.isdir(path) and os.path.exists(os.path.join(path, "config.json"))


def read_spec(path: str):
    """(StackSpec, SafetensorsFile) of a model folder."""
    from .designs import DESIGNS
    from .safetensors import SafetensorsFile
    with open(os.path.join(path, "config.json"), encoding="utf-8") as f:
        cfg = json.load(f)
    name = cfg.get("architecture")
    if name not in DESIGNS:
        raise ValueError(f"{path}: architecture {name!r} is not known (known: {', '.join(sorted(DESIGNS))})")
    weights = SafetensorsFile(os.path.join(path, "model.safetensors"))
    return DESIGNS[name](cfg, weights.shape), weights


def load_model(path: str, device: int = 0, max_streams: int = 1, dtype: str = "bfloat16", seq_len: int = 0, max_step_tokens: int = 0,
               flags: int = 0, verbose: bool = False, build: bool = False) -> HipModel:
    """Any model by path.  dtype / seq_len / max_step_tokens apply to layer-stack designs; build: compile the family's library
    first if it is missing or older than its sources."""
    if is_model_folder(path):
        from .stack import load_stack_model
        spec, weights = read_spec(path)
        if build:
            _lib.build(family="stack")
        return load_stack_model(spec, weights.get, device, max_streams, seq_len, dtype, max_step_tokens, flags, verbose)
    from .gguf import load_gguf
    from .model import load_llama_model
    if build:
        _lib.build()
    return load_llama_model(load_gguf(path, verbose=verbose), device=device, max_streams=max_streams, flags=flags, verbose=verbose)
