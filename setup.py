"""Build the helix_amd native extension in-tree for MI355X (gfx950).

Usage: PYTORCH_ROCM_ARCH=gfx950 python setup.py build_ext --inplace
"""
import os
import glob
from setuptools import setup

os.environ.setdefault("PYTORCH_ROCM_ARCH", "gfx950")

from torch.utils.cpp_extension import BuildExtension, CUDAExtension  # noqa: E402

ROOT = os.path.dirname(os.path.abspath(__file__))
HIP_DIR = os.path.join(ROOT, "helix_amd", "ops", "hip")

# Packed-fp32 VALU forms (v_pk_{add,mul,fma}_f32) stay off: hipcc -O3 forms
# them from ordinary float code and some have given wrong results here.
NO_PACKED_FP32 = ["-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]

sources = sorted(
    f for f in glob.glob(os.path.join(HIP_DIR, "*.hip"))
    if not f.endswith("_hip.hip")       # torch-hipify build artifacts
) + [os.path.join(HIP_DIR, "bindings.cpp")]

setup(
    name="helix_amd_C",
    ext_modules=[
        CUDAExtension(
            name="helix_amd._C",
            sources=sources,
            extra_compile_args={
                "cxx": ["-O3", "-std=c++17"],
                "nvcc": ["-O3", "-std=c++17"] + NO_PACKED_FP32,
            },
        )
    ],
    cmdclass={"build_ext": BuildExtension},
)
