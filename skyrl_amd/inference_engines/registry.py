"""Model registry: a checkpoint folder (config.json + safetensors) -> decoder.

config.json names its design either as `architecture` (designs of this framework) or, in an HF
checkpoint, as `model_type`."""

from __future__ import annotations

import glob
import json
import os
from typing import Any, Callable, Dict, Iterator, Optional, Tuple

import torch


def _hybrid(config: Dict[str, Any], folder: str, device, dtype, max_model_len, seed):
    from .hybrid import HybridDecoder

    return HybridDecoder(config, device, dtype=dtype, seed=seed, max_model_len=max_model_len)


def _hf_paged(config: Dict[str, Any], folder: str, device, dtype, max_model_len, seed):
    from transformers import AutoConfig

    from .model import PagedDecoder

    if dtype != torch.bfloat16:
        raise ValueError("the paged HF decoders run in bfloat16")
    return PagedDecoder(AutoConfig.from_pretrained(folder), device, dtype=dtype, seed=seed,
                        max_model_len=max_model_len)


ARCHITECTURES: Dict[str, Callable] = {"Dovidra": _hybrid, "Lipedra": _hybrid, "Foduzen": _hybrid, "Tativik": _hybrid}
HF_MODEL_TYPES: Dict[str, Callable] = {t: _hf_paged for t in ("qwen2", "llama", "mistral", "qwen3")}


def read_config(folder: str) -> Dict[str, Any]:
    with open(os.path.join(folder, "config.json")) as f:
        return json.load(f)


def decoder_factory(config: Dict[str, Any]) -> Callable:
    arch, mt = config.get("architecture"), config.get("model_type")
    if arch is not None:
        if arch not in ARCHITECTURES:
            raise ValueError(f"unknown architecture {arch!r} (known: {sorted(ARCHITECTURES)})")
        return ARCHITECTURES[arch]
    if mt not in HF_MODEL_TYPES:
        raise ValueError(f"unsupported model_type {mt!r} (known: {sorted(HF_MODEL_TYPES)})")
    return HF_MODEL_TYPES[mt]


def build_decoder(config: Dict[str, Any], device, dtype: torch.dtype = torch.bfloat16,
                  max_model_len: Optional[int] = None, seed: Optional[int] = 0, folder: str = ""):
    """A decoder with random (seed) or zeroed (None) weights."""
    return decoder_factory(config)(config, folder, device, dtype, max_model_len, seed)


def kernel_libraries(config: Dict[str, Any]) -> Tuple[str, ...]:
    """The layer libraries (_ffi.LAYER_LIBS) that serving the checkpoint needs; none for the paged HF decoders."""
    if decoder_factory(config) is not _hybrid:
        return ()
    from .hybrid import DESIGNS
    from .mixers import MIXERS

    unknown = sorted({e["type"] for e in config["layers"]} - set(MIXERS))
    if unknown:
        raise ValueError(f"unknown layer types {unknown} (known: {sorted(MIXERS)})")
    ffs = DESIGNS[config["architecture"]].feedforwards
    kinds = [MIXERS[e["type"]] for e in config["layers"]] + [ffs[e["mlp"]["kind"]] for e in config["layers"]
                                                             if e.get("mlp") and e["mlp"]["kind"] in ffs]
    return ("layers",) + tuple(sorted({lib for k in kinds for lib in getattr(k, "libraries", ())}))


def checkpoint_tensors(folder: str) -> Iterator[Tuple[str, torch.Tensor]]:
    from safetensors import safe_open

    files = sorted(glob.glob(os.path.join(folder, "*.safetensors")))
    if not files:
        raise FileNotFoundError(f"no .safetensors file in {folder}")
    for path in files:
        with safe_open(path, framework="pt", device="cpu") as f:
            for name in f.keys():
                yield name, f.get_tensor(name)


def checkpoint_shapes(folder: str) -> Dict[str, Tuple[int, ...]]:
    """Every tensor's shape, from the files' headers."""
    from safetensors import safe_open

    out: Dict[str, Tuple[int, ...]] = {}
    for path in sorted(glob.glob(os.path.join(folder, "*.safetensors"))):
        with safe_open(path, framework="pt", device="cpu") as f:
            out.update((name, tuple(f.get_slice(name).get_shape())) for name in f.keys())
    return out


def complete_config(config: Dict[str, Any], folder: str) -> Dict[str, Any]:
    """The config with the sizes that its mechanisms take from the checkpoint's tensors."""
    if decoder_factory(config) is not _hybrid:
        return config
    from .mixers import MIXERS

    shapes, layers = None, list(config["layers"])
    for i, e in enumerate(layers):
        complete = getattr(MIXERS.get(e["type"]), "complete", None)
        if complete is not None:
            shapes = checkpoint_shapes(folder) if shapes is None else shapes
            layers[i] = dict(e, mixer=complete(e["mixer"], lambda name: shapes.get(f"l{i}.mix.{name}")))
    return dict(config, layers=layers)


def load_decoder(folder: str, device, dtype: torch.dtype = torch.bfloat16, max_model_len: Optional[int] = None):
    """The checkpoint's decoder with its weights loaded; a checkpoint that lacks a parameter is an error."""
    config = complete_config(read_config(folder), folder)
    model = build_decoder(config, device, dtype, max_model_len, seed=None, folder=folder)
    seen = set()

    def named():
        for name, t in checkpoint_tensors(folder):
            seen.add(name)
            yield name, t

    model.load_weights(named())
    missing = sorted(n for n, _ in model.hf_named_tensors() if n not in seen)
    if missing:
        raise ValueError(f"checkpoint {folder} lacks {missing[:5]}{'...' if len(missing) > 5 else ''}")
    return model
