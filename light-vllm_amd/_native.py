"""Loader of the native libraries.  No fallback: if a HIP library or a torch
binding is missing or fails to load, importing this module's users raises, so a product
path can never silently run on something else.

The libraries come in components (build.py): "base" is what every model needs, "full" includes all the others.
`limit_to(components)`, called before anything else of the package is imported, makes a process that serves one model load
(and need) that model's components alone."""
import ctypes
import os

import torch  # must be first: its HIP runtime (same SONAME) is the one the kernels use

from .build import ALL, COMPONENTS, LIBDIR, with_needed

LIB_PATH = os.path.join(LIBDIR, COMPONENTS["full"][1])
EXT_PATH = os.path.join(LIBDIR, COMPONENTS["full"][3])

_state = {"lib": None, "ext": False, "components": ALL}


class NativeLibraryError(ImportError):
    pass


def limit_to(components) -> None:
    """This process serves a model that these components cover: nothing else is loaded or required."""
    if _state["lib"] is not None or _state["ext"]:
        raise NativeLibraryError("limit_to() must come before the native libraries are loaded")
    _state["components"] = with_needed(components)


def _require(path: str) -> str:
    if not os.path.exists(path):
        raise NativeLibraryError(
            f"{path} not found: build it with `python -c 'import __graft_entry__ as g; g.build()'` "
            "(hipcc --offload-arch=gfx950); there is no CPU fallback")
    return path


def load_hip_library() -> ctypes.CDLL:
    """ctypes handle on the C-ABI (include/lvllm_hip.h); with fewer than all components, on the last of them."""
    if _state["lib"] is None:
        for c in _state["components"]:
            lib = ctypes.CDLL(_require(os.path.join(LIBDIR, COMPONENTS[c][1])), mode=ctypes.RTLD_GLOBAL)
        lib.lvllm_last_error.restype = ctypes.c_char_p
        lib.lvllm_version.restype = ctypes.c_char_p
        _state["lib"] = lib
    return _state["lib"]


def load_torch_ops() -> None:
    """Registers torch.ops._C / _C_cache_ops / _C_cuda_utils (reference schemas) and _C_amd."""
    if not _state["ext"]:
        load_hip_library()
        for c in _state["components"]:
            torch.ops.load_library(_require(os.path.join(LIBDIR, COMPONENTS[c][3])))
        _state["ext"] = True


def loaded_libraries():
    last = COMPONENTS[_state["components"][-1]]
    return {"hip": os.path.join(LIBDIR, last[1]) if _state["lib"] is not None else None,
            "torch_ops": os.path.join(LIBDIR, last[3]) if _state["ext"] else None}
