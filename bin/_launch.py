"""What the programs of this folder share: the repository on the import path, and the native components a model needs,
compiled where they are missing or older than their sources."""
import os
import sys

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def prepare(model_dir: str):
    """Returns the model's registry entry, with its native libraries built and the loader told which ones it needs."""
    sys.path.insert(0, ROOT)
    import light_vllm_amd  # noqa: F401
    from light_vllm_amd import _native
    from light_vllm_amd import build
    from light_vllm_amd.engine.registry import model_entry, read_architecture
    entry = model_entry(read_architecture(model_dir))
    build.build_all(entry.native)
    _native.limit_to(entry.native)
    return entry


DTYPES = ("bfloat16", "float32")


def torch_dtype(name: str):
    import torch
    if name == "float32":  # true 32-bit products
        torch.backends.cuda.matmul.allow_tf32 = False
        torch.set_float32_matmul_precision("highest")
    return {"bfloat16": torch.bfloat16, "float32": torch.float32}[name]
