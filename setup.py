"""In-tree build of the mdi_llm_amd HIP extension for gfx950 (MI355X).

Two-step build, fully controlled (no hipify, no JIT cache):
  1. hipcc compiles the .hip kernel TUs with --offload-arch=gfx950
     (device code; no torch headers needed).
  2. the host bindings TU is built as a plain C++ torch extension and
     linked with the kernel objects + libamdhip64.

Usage:  python setup.py build_ext --inplace
The resulting mdi_llm_amd/_hip_ops*.so ships with the repo snapshot to the
GPU box (it is git-ignored).
"""

import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor
from pathlib import Path

from setuptools import setup
from torch.utils.cpp_extension import BuildExtension, CppExtension
import torch

ROOT = Path(__file__).resolve().parent
HIP_DIR = ROOT / "mdi_llm_amd" / "ops" / "hip"
BUILD_DIR = ROOT / "build" / "hip_objs"

ROCM_HOME = os.environ.get("ROCM_HOME", os.environ.get("ROCM_PATH", "/opt/rocm"))
HIPCC = os.path.join(ROCM_HOME, "bin", "hipcc")
OFFLOAD_ARCH = os.environ.get("PYTORCH_ROCM_ARCH", "gfx950").split(";")[0]

KERNEL_SOURCES = ["decode_kernels.hip", "hybrid_kernels.hip",
                  "paged_attn_bf16.hip", "paged_attn_f32.hip",
                  "diff_attn_bf16.hip", "diff_attn_f32.hip",
                  "slope_attn_bf16.hip", "slope_attn_f32.hip",
                  "row_attn_bf16.hip", "row_attn_f32.hip",
                  "latent_kernels.hip", "moe_kernels.hip",
                  "recurrent_kernels.hip", "mlstm_kernels.hip",
                  "stream_kernels.hip", "skinny_gemm.hip"]
HEADERS = [HIP_DIR / h for h in ("decode_kernels.h", "hybrid_kernels.h",
                                 "hybrid_common.h", "mfma_frag.h",
                                 "mfma_tile.h", "matrix_state.h",
                                 "paged_attn.inc", "row_attn.inc")]


def compile_one(src: str) -> str:
    src_path = HIP_DIR / src
    obj_path = BUILD_DIR / (src_path.stem + ".o")
    inputs = [src_path, Path(__file__), *HEADERS]
    # MDI_FORCE_BUILD=1: compile whatever the dates say
    if os.environ.get("MDI_FORCE_BUILD") == "1" or not obj_path.exists() or any(
        obj_path.stat().st_mtime < p.stat().st_mtime for p in inputs
    ):
        cmd = [
            HIPCC,
            f"--offload-arch={OFFLOAD_ARCH}",
            "-O3",
            "-std=c++17",
            "-fPIC",
            # the packed fp32 instructions are not reliable on this part
            "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
            "-c",
            str(src_path),
            "-o",
            str(obj_path),
        ]
        print("[hipcc]", " ".join(cmd), flush=True)
        subprocess.check_call(cmd)
    return str(obj_path)


def compile_hip_objects() -> list:
    BUILD_DIR.mkdir(parents=True, exist_ok=True)
    with ThreadPoolExecutor(max_workers=8) as pool:
        return list(pool.map(compile_one, KERNEL_SOURCES))


HIP_OBJECTS = compile_hip_objects()


def torch_lib_dir() -> str:
    return str(Path(torch.__file__).parent / "lib")


ext = CppExtension(
    name="mdi_llm_amd._hip_ops",
    sources=[str(HIP_DIR / "bindings.cpp"),
             str(HIP_DIR / "hybrid_bindings.cpp")],
    extra_objects=HIP_OBJECTS,
    # relink when an object changes, not only when the bindings do
    depends=[*HIP_OBJECTS, *map(str, HEADERS)],
    include_dirs=[os.path.join(ROCM_HOME, "include")],
    library_dirs=[os.path.join(ROCM_HOME, "lib"), torch_lib_dir()],
    libraries=["amdhip64", "c10_hip", "torch_hip"],
    extra_compile_args=["-D__HIP_PLATFORM_AMD__=1", "-O2"],
)

setup(
    name="mdi_llm_amd_ops",
    version="0.1.0",
    ext_modules=[ext],
    cmdclass={"build_ext": BuildExtension.with_options(no_python_abi_suffix=False)},
)
