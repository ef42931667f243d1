"""Model registry: what serves a configuration (model class, attention backend, native component) and how a model folder
becomes a configuration.  Entries import lazily, so that a process serving one model loads that model's code and native
libraries only."""
import json
import os
from dataclasses import dataclass
from importlib import import_module
from typing import Tuple

import torch


def _load(path: str):
    module, name = path.split(":")
    return getattr(import_module(module, __package__), name)


@dataclass(frozen=True)
class ModelEntry:
    config: str                     # "module:class"; a config class with from_dict reads a model folder's config.json
    model: str                      # forward / compute_logits / greedy_tokens
    backend: str                    # attention backend: metadata, cache shapes, block movement
    native: Tuple[str, ...]         # components of build.py the model's kernels live in

    def model_cls(self):
        return _load(self.model)

    def backend_cls(self):
        return _load(self.backend)

    def config_cls(self):
        return _load(self.config)


MODELS = {
    # Llama / Qwen2-shaped decoders (random weights: engine/config.py ModelConfig)
    "RotaryDecoder": ModelEntry(".config:ModelConfig", ".model:DecoderModel", "..attention.backend:PagedAttnBackend",
                                ("full",)),
    "Sasilorn": ModelEntry(".hybrid_config:HybridModelConfig", ".hybrid_model:HybridModel",
                           "..attention.head_backend:HeadAttnBackend", ("heads", "hybrid")),
    "Lepalorn": ModelEntry(".latent_config:LatentModelConfig", ".latent_model:LatentModel",
                           "..attention.latent_backend:LatentAttnBackend", ("heads", "moe", "latent")),
    "Lizazen": ModelEntry(".local_config:LocalModelConfig", ".local_model:LocalModel",
                          "..attention.head_backend:HeadAttnBackend", ("heads", "moe", "local")),
    "Susalorn": ModelEntry(".stream_config:StreamModelConfig", ".stream_model:StreamModel",
                           "..attention.latent_backend:LatentAttnBackend", ("heads", "moe", "latent", "delta")),
}


def model_entry(architecture: str) -> ModelEntry:
    try:
        return MODELS[architecture]
    except KeyError:
        raise ValueError(f"unknown architecture {architecture!r} (known: {', '.join(sorted(MODELS))})") from None


def read_architecture(model_dir: str) -> str:
    with open(os.path.join(model_dir, "config.json")) as f:
        return json.load(f)["architecture"]


def load_model_config(model_dir: str, dtype: torch.dtype = torch.bfloat16):
    """The configuration of a model folder (config.json + model.safetensors), by its `architecture`."""
    with open(os.path.join(model_dir, "config.json")) as f:
        c = json.load(f)
    cls = model_entry(c["architecture"]).config_cls()
    if not hasattr(cls, "from_dict"):
        raise ValueError(f"{c['architecture']} models are not loaded from a folder")
    return cls.from_dict(c, dtype=dtype, weights_dir=model_dir)
