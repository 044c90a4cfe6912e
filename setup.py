"""In-tree build of the rbg_amd HIP extensions for gfx950 (MI355X).

Usage: PYTORCH_ROCM_ARCH=gfx950 python setup.py build_ext --inplace
The resulting rbg_amd/ops/_hip_*.so travel with the repo snapshot to GPU
boxes (no JIT cache involved).

The extensions and their sources are listed in rbg_amd/utils/hip_build.py;
RBG_BUILD_EXT=<name>[,<name>] restricts the build to some of them.
"""
import os
import sys

from setuptools import setup

os.environ.setdefault("PYTORCH_ROCM_ARCH", "gfx950")

from torch.utils.cpp_extension import BuildExtension, CUDAExtension  # noqa: E402

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
from rbg_amd.utils.hip_build import HIP_SOURCES  # noqa: E402

HIP_DIR = os.path.join("rbg_amd", "ops", "hip")

# no packed-f32 VALU instructions: some of their forms are unreliable here
NVCC_ARGS = ["-O3", "-std=c++17", "--offload-arch=gfx950",
             "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]

only = [n for n in os.environ.get("RBG_BUILD_EXT", "").split(",") if n]
ext_modules = [
    CUDAExtension(
        name=f"rbg_amd.ops.{name}",
        sources=[os.path.join(HIP_DIR, f) for f in files],
        extra_compile_args={"cxx": ["-O3", "-std=c++17"], "nvcc": NVCC_ARGS},
    )
    for name, files in HIP_SOURCES.items() if not only or name in only]

setup(
    name="rbg-mi355x",
    version="0.1.0",
    packages=["rbg_amd"],
    ext_modules=ext_modules,
    cmdclass={"build_ext": BuildExtension.with_options(use_ninja=True)},
)
