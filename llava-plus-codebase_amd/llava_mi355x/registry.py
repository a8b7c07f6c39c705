"""Model families of the package and the choice between them by a checkpoint folder's config.json.

    family_of(path)                 the family's entry
    load_model(path, dtype=...)     config + weights -> a model (an EngineCausalLM)

A family is found by config.json's `architecture`, the first of `architectures`, or `model_type`."""
from __future__ import annotations

import glob
import importlib
import json
import os
from dataclasses import dataclass
from typing import Dict, Iterator, Tuple

import torch


def iter_checkpoint(path: str) -> Iterator[Tuple[str, torch.Tensor]]:
    """Yield (key, tensor) from every weight shard in a HF-format directory (or a single file)."""
    files = [path] if os.path.isfile(path) else sorted(glob.glob(os.path.join(path, "*.safetensors")))
    if not files:
        files = sorted(glob.glob(os.path.join(path, "pytorch_model*.bin")))
    if not files:
        raise FileNotFoundError(f"no *.safetensors / pytorch_model*.bin under {path}")
    for f in files:
        if f.endswith(".safetensors"):
            from safetensors import safe_open
            with safe_open(f, framework="pt", device="cpu") as sf:
                for k in sf.keys():
                    yield k, sf.get_tensor(k)
        else:
            try:
                sd = torch.load(f, map_location="cpu", mmap=True, weights_only=True)
            except (RuntimeError, ValueError):          # legacy (non-zip) .bin shards cannot be memory-mapped; the reference loads them too
                sd = torch.load(f, map_location="cpu", weights_only=True)
            for k, v in sd.items():
                yield k, v


def checkpoint_shapes(path: str) -> Dict[str, Tuple[int, ...]]:
    """{key: shape} of a directory's *.safetensors, from their headers alone."""
    from safetensors import safe_open
    out: Dict[str, Tuple[int, ...]] = {}
    for f in sorted(glob.glob(os.path.join(path, "*.safetensors"))):
        with safe_open(f, framework="pt", device="cpu") as sf:
            for k in sf.keys():
                out[k] = tuple(sf.get_slice(k).get_shape())
    return out


@dataclass(frozen=True)
class ModelFamily:
    name: str
    module: str                      # module of this package, imported when the family is used
    loader: str                      # "Class.method" or function there: (path, torch_dtype=, device=, max_position=) -> model
    multimodal: bool = False

    def load(self, path: str, **kw):
        obj = importlib.import_module(f".{self.module}", __package__)
        for part in self.loader.split("."):
            obj = getattr(obj, part)
        return obj(path, **kw)


FAMILIES: Dict[str, ModelFamily] = {}


def register(family: ModelFamily, *keys: str) -> None:
    for k in keys:
        FAMILIES[k.lower()] = family


register(ModelFamily("llava", "builder", "from_pretrained", multimodal=True), "llava", "LlavaLlamaForCausalLM")
register(ModelFamily("siterax", "siterax", "SiteraxForCausalLM.from_pretrained"), "siterax", "SiteraxForCausalLM")
register(ModelFamily("vizosun", "vizosun", "VizosunForCausalLM.from_pretrained"), "vizosun", "VizosunForCausalLM")


def family_of(path: str) -> ModelFamily:
    with open(os.path.join(path, "config.json")) as f:
        c = json.load(f)
    keys = [k for k in (c.get("architecture"), (c.get("architectures") or [None])[0], c.get("model_type")) if k]
    for k in keys:
        if str(k).lower() in FAMILIES:
            return FAMILIES[str(k).lower()]
    raise ValueError(f"{path}: no model family for {keys or 'a config.json without architecture / architectures / model_type'} (known: {sorted(FAMILIES)})")


def load_model(path: str, dtype: torch.dtype = torch.bfloat16, device="cuda", max_position=None):
    return family_of(path).load(path, torch_dtype=dtype, device=device, max_position=max_position)
