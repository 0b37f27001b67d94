"""In-tree compilation of the HIP kernel libraries (hipcc, gfx950).

Two libraries, each a torch extension next to this file:

- ``_hip_ops.so``: every kernel in ``csrc/*.hip`` (vision, encoder and
  llama/gpt2 serving)
- ``_hip_lm.so``: the token-batch kernels in ``csrc/lm/*.hip`` (latent
  attention, gated linear recurrence, norms and the residual stream) plus
  the decode GEMM they share with ``_hip_ops``. It is a library of its own so that a
  fresh checkout can serve a model of that kind after compiling only this.
"""

import glob
import os
import shutil
from typing import List

OPS_DIR = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(OPS_DIR, "csrc")

# Packed FP32 arithmetic stays off: some v_pk_*_f32 forms have returned wrong
# results on gfx950. The host pass warns about the unknown feature; harmless.
HIP_FLAGS = ["-O3", "-std=c++17",
             "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]
CXX_FLAGS = ["-O3", "-std=c++17"]


def _sources(name: str) -> List[str]:
    if name == "_hip_ops":
        pats = ["*.hip", "*.cpp"]
    elif name == "_hip_lm":
        pats = ["lm/*.hip", "lm/*.cpp", "skinny_gemm.hip"]
    else:
        raise ValueError("unknown kernel library '{}'".format(name))
    out: List[str] = []
    for p in pats:
        out += [g for g in glob.glob(os.path.join(CSRC, p))
                if not g.endswith("_hip.hip")]
    return sorted(out)


def so_path(name: str) -> str:
    return os.path.join(OPS_DIR, name + ".so")


def build_library(name: str, verbose: bool = True) -> str:
    """Compile one library from source, always (no reuse of old objects)."""
    os.environ.setdefault("PYTORCH_ROCM_ARCH", "gfx950")
    import torch  # noqa: F401  (sets up the extension toolchain)
    from torch.utils.cpp_extension import load

    # torch's hipify writes generated *_hip.hip siblings into csrc and SKIPS
    # regeneration when they already exist -- stale copies silently shadow
    # edited kernels, so delete them before every build
    for pat in ("*_hip.hip", os.path.join("lm", "*_hip.hip")):
        for stale in glob.glob(os.path.join(CSRC, pat)):
            os.remove(stale)
    build_dir = os.path.join(OPS_DIR, "build", name)
    shutil.rmtree(build_dir, ignore_errors=True)
    os.makedirs(build_dir)
    load(name=name, sources=_sources(name), extra_cflags=CXX_FLAGS,
         extra_cuda_cflags=HIP_FLAGS, build_directory=build_dir,
         verbose=verbose, is_python_module=False, is_standalone=False)
    out = so_path(name)
    tmp = out + ".tmp{}".format(os.getpid())
    shutil.copy2(os.path.join(build_dir, name + ".so"), tmp)
    os.replace(tmp, out)  # readers never see a half-written library
    return out


def ensure_library(name: str) -> str:
    """Compile ``name`` only if it is not there yet."""
    out = so_path(name)
    return out if os.path.exists(out) else build_library(name)
