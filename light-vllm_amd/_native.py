"""Loader of the native libraries.  No fallback: if a HIP library or a torch
binding is missing or fails to load, importing this module's users raises, so a product
path can never silently run on something else.

Two components (build.py): "base" -- what every model needs -- and "full" -- base plus the operators of the rotary
decoders.  `limit_to_base()`, called before anything else of the package is imported, makes a process that serves a
base-only model load (and need) the first alone."""
import ctypes
import os

import torch  # must be first: its HIP runtime (same SONAME) is the one the kernels use

_LIBDIR = os.path.join(os.path.dirname(os.path.abspath(__file__)), "lib")
BASE_LIB_PATH = os.path.join(_LIBDIR, "liblvllm_base.so")
BASE_EXT_PATH = os.path.join(_LIBDIR, "_C_base.so")
LIB_PATH = os.path.join(_LIBDIR, "liblvllm_hip.so")
EXT_PATH = os.path.join(_LIBDIR, "_C.so")

_state = {"lib": None, "ext": False, "base_only": False}


class NativeLibraryError(ImportError):
    pass


def limit_to_base() -> None:
    """This process serves a model that the base component alone covers: nothing else is loaded or required."""
    if _state["lib"] is not None or _state["ext"]:
        raise NativeLibraryError("limit_to_base() must come before the native libraries are loaded")
    _state["base_only"] = True


def _require(path: str) -> str:
    if not os.path.exists(path):
        raise NativeLibraryError(
            f"{path} not found: build it with `python -c 'import __graft_entry__ as g; g.build()'` "
            "(hipcc --offload-arch=gfx950); there is no CPU fallback")
    return path


def load_hip_library() -> ctypes.CDLL:
    """ctypes handle on the C-ABI (include/lvllm_hip.h)."""
    if _state["lib"] is None:
        lib = ctypes.CDLL(_require(BASE_LIB_PATH), mode=ctypes.RTLD_GLOBAL)
        if not _state["base_only"]:
            lib = ctypes.CDLL(_require(LIB_PATH), mode=ctypes.RTLD_GLOBAL)
        lib.lvllm_last_error.restype = ctypes.c_char_p
        lib.lvllm_version.restype = ctypes.c_char_p
        _state["lib"] = lib
    return _state["lib"]


def load_torch_ops() -> None:
    """Registers torch.ops._C / _C_cache_ops / _C_cuda_utils (reference schemas) and _C_amd."""
    if not _state["ext"]:
        load_hip_library()
        for path in [BASE_EXT_PATH] + ([] if _state["base_only"] else [EXT_PATH]):
            torch.ops.load_library(_require(path))
        _state["ext"] = True


def loaded_libraries():
    full = not _state["base_only"]
    return {"hip": (LIB_PATH if full else BASE_LIB_PATH) if _state["lib"] is not None else None,
            "torch_ops": (EXT_PATH if full else BASE_EXT_PATH) if _state["ext"] else None}
