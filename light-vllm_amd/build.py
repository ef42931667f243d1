"""Build the gfx950 native libraries in-tree (no cmake, no hipify), in components:

  base    what every model needs: error plumbing, cache block movement, the weight-streaming GEMMs of decode steps, step
          inputs, the sampler
  heads   softmax attention over paged caches of unequal key and value sizes, and what goes into them
  moe     routers and grouped products of mixtures of experts
  hybrid  row-wise operators and recurrences of the hybrid decoders
  latent  latent attention, norms on sublayer outputs and depth averages
  local   retention, norms around sublayers, embeddings of token pairs (local decoders)
  delta   residual streams, short convolutions, the gated delta rule (stream decoders)
  full    the rest of the C-ABI of include/lvllm_hip.h (paged and prefill attention of the rotary decoders, norms, fp8); it
          needs all the others, so a handle on liblvllm_hip.so resolves every symbol of the header

Each is a kernel library (hipcc --offload-arch=gfx950, one object per .hip, linked -shared) and a torch extension: op
registrations (`torch.ops._C`, `_C_cache_ops`, `_C_cuda_utils`, `_C_amd`) forwarding to the C-ABI; host-only C++, built with
g++ against the torch headers.

`build_all(("base", "latent"))` builds what a model whose registry entry says so will load.
All land in light-vllm_amd/lib/.  Objects are cached under build/ keyed on the
source mtime, so a rebuild after touching one kernel takes seconds.
"""
import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

PKG = os.path.dirname(os.path.abspath(__file__))
ROOT = os.path.dirname(PKG)
CSRC = os.path.join(PKG, "csrc")
LIBDIR = os.path.join(PKG, "lib")
OBJDIR = os.path.join(ROOT, "build", "obj")
ARCH = "gfx950"

SOURCES = {
    "base": ["capi.hip", "cache.hip", "skinny_gemm.hip", "prepare_inputs.hip", "sampler.hip", "activation.hip"],
    "heads": ["head_attention.hip", "head_attention_prefill.hip", "head_attention_decode.hip", "head_attention_maps.hip",
              "head_cache.hip"],
    "moe": ["moe.hip", "moe_mfma.hip"],
    "hybrid": ["token_mix.hip", "recurrent.hip"],
    "latent": ["latent_attention.hip", "latent_attention_mfma.hip", "depth_mix.hip"],
    "local": ["retention.hip", "sandwich_norm.hip"],
    "delta": ["delta_rule.hip", "short_conv.hip", "stream_mix.hip"],
    "full": ["layernorm.hip", "pos_encoding.hip", "attention.hip", "attention_bf16.hip", "attention_f16.hip",
             "prefill_attention.hip", "fp8_quant.hip"],
}
ALL = tuple(SOURCES)  # in link order: "base" is needed by the others, "full" needs all
# component -> (sources, kernel library, torch registrations, torch extension)
COMPONENTS = {c: (src,) + (("liblvllm_hip.so", "torch_bindings.cpp", "_C.so") if c == "full" else
                           (f"liblvllm_{c}.so", f"torch_bindings_{c}.cpp", f"_C_{c}.so"))
              for c, src in SOURCES.items()}


def with_needed(components):
    """The components and what they need, in link order."""
    return ALL if "full" in components else tuple(c for c in ALL if c == "base" or c in components)


def _links(component):
    """Linker flags for the kernel libraries a component's own kernel library needs."""
    need = [] if component == "base" else [c for c in ALL if c != "full"] if component == "full" else ["base"]
    return (["-L", LIBDIR] + [f"-llvllm_{c}" for c in need] + ["-Wl,-rpath,$ORIGIN"]) if need else []


HIPCC = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
# tuning experiments: e.g. LVLLM_EXTRA_HIPCC_FLAGS="-DLVLLM_ATTN_NBUF=2 -DLVLLM_ATTN_TUNE_ONLY"
# No packed fp32 arithmetic (v_pk_add / mul / fma_f32): some of its forms have given wrong results on this hardware.
BASE_FLAGS = ["-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]
EXTRA_FLAGS = os.environ.get("LVLLM_EXTRA_HIPCC_FLAGS", "").split()


def _newer(target, deps):
    if not os.path.exists(target):
        return True
    t = os.path.getmtime(target)
    return any(os.path.getmtime(d) > t for d in deps)


def _headers():
    hs = [os.path.join(CSRC, f) for f in os.listdir(CSRC) if f.endswith(".h")]
    hs.append(os.path.join(ROOT, "include", "lvllm_hip.h"))
    return hs


def _run(cmd):
    r = subprocess.run(cmd, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)
    if r.returncode != 0:
        raise RuntimeError("command failed: %s\n%s" % (" ".join(cmd), r.stdout))
    return r.stdout


# Per-source flags.  The prefill kernel's softmax is vector-issue bound; without NaN honouring the
# compiler drops the canonicalising v_max x,x,x it otherwise puts in front of every max of an
# MFMA result (3 instructions per max -> 1).  Masked / out-of-range keys are removed by selects,
# not by NaN propagation, so results on finite data are unchanged.
PER_SOURCE_FLAGS = {"prefill_attention.hip": ["-fno-honor-nans"]}


def build_kernels(components=ALL, verbose=False, force=False):
    os.makedirs(OBJDIR, exist_ok=True)
    os.makedirs(LIBDIR, exist_ok=True)
    hdrs = _headers()
    jobs = []
    objs = {c: [] for c in components}
    for c in components:
        for src in COMPONENTS[c][0]:
            s = os.path.join(CSRC, src)
            o = os.path.join(OBJDIR, src.replace(".hip", ".o"))
            objs[c].append(o)
            if force or _newer(o, [s] + hdrs):
                jobs.append([HIPCC, "--offload-arch=" + ARCH, "-O3", "-std=c++17", "-fPIC",
                             "-ffp-contract=off", "-Wall", "-Wno-unused-function"] + BASE_FLAGS +
                            PER_SOURCE_FLAGS.get(src, []) + EXTRA_FLAGS + ["-c", s, "-o", o])
    if jobs:
        with ThreadPoolExecutor(max_workers=min(6, len(jobs))) as ex:
            for out in ex.map(_run, jobs):
                if verbose and out.strip():
                    print(out)
    libs = []
    for c in components:
        lib = os.path.join(LIBDIR, COMPONENTS[c][1])
        libs.append(lib)
        if force or _newer(lib, objs[c] + [os.path.abspath(__file__)]):
            # no rpath to /opt/rocm on purpose: inside a torch process the HIP
            # runtime torch already loaded (same SONAME) must be the one used.
            _run([HIPCC, "--offload-arch=" + ARCH, "-shared", "-fPIC", "-o", lib] + objs[c] +
                 (["-Wl,--no-as-needed"] + _links(c) if c == "full" else _links(c)))
    return libs


def build_torch_bindings(components=ALL, verbose=False, force=False):
    import torch  # noqa: F401  (header + library locations)
    from torch.utils import cpp_extension as ce
    import sysconfig

    os.makedirs(LIBDIR, exist_ok=True)
    incs = ce.include_paths("cuda") + [sysconfig.get_paths()["include"], os.path.join(ROOT, "include")]
    torch_lib = os.path.join(os.path.dirname(torch.__file__), "lib")
    hdrs = [os.path.join(CSRC, "torch_bindings.h"), os.path.join(ROOT, "include", "lvllm_hip.h")]
    jobs, outs = [], []
    for c in components:
        src = os.path.join(CSRC, COMPONENTS[c][2])
        name = COMPONENTS[c][3]
        out = os.path.join(LIBDIR, name)
        outs.append(out)
        if not force and not _newer(out, [src] + hdrs):
            continue
        cmd = ["g++", "-O2", "-std=c++17", "-fPIC", "-shared", "-D__HIP_PLATFORM_AMD__=1",
               "-DUSE_ROCM=1", "-DTORCH_EXTENSION_NAME=" + name[:-3],
               "-D_GLIBCXX_USE_CXX11_ABI=%d" % int(torch._C._GLIBCXX_USE_CXX11_ABI),
               "-Wno-deprecated-declarations"]
        for i in incs:
            cmd += ["-I", i]
        jobs.append(cmd + [src, "-o", out, "-L", torch_lib, "-L", LIBDIR,
                           "-ltorch", "-ltorch_cpu", "-ltorch_hip", "-lc10", "-lc10_hip"] +
                    ["-llvllm_hip" if c == "full" else f"-llvllm_{c}", "-llvllm_base", "-Wl,-rpath,$ORIGIN"])
    if jobs:
        with ThreadPoolExecutor(max_workers=len(jobs)) as ex:
            for o in ex.map(_run, jobs):
                if verbose and o.strip():
                    print(o)
    return outs


def build_all(components=ALL, verbose=False, force=False):
    """(kernel libraries, torch extensions) of the components, built where they are missing or older than a source
    (`force`: all of them)."""
    components = with_needed(components)
    return build_kernels(components, verbose, force), build_torch_bindings(components, verbose, force)


if __name__ == "__main__":
    print(build_all(verbose="-v" in sys.argv))
