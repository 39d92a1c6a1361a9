"""Build the helix_amd native extensions in-tree for MI355X (gfx950).

Usage: PYTORCH_ROCM_ARCH=gfx950 python setup.py build_ext --inplace

HELIX_BUILD_ONLY (comma-separated module names, e.g. "_C_ext") limits the
build to the extensions one model needs.
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


def extension(name, folder):
    sources = sorted(
        f for f in glob.glob(os.path.join(folder, "*.hip"))
        if not f.endswith("_hip.hip")       # torch-hipify build artifacts
    ) + [os.path.join(folder, "bindings.cpp")]
    return CUDAExtension(
        name=f"helix_amd.{name}",
        sources=sources,
        extra_compile_args={
            "cxx": ["-O3", "-std=c++17"],
            "nvcc": ["-O3", "-std=c++17"] + NO_PACKED_FP32,
        },
    )


EXTENSIONS = {"_C": HIP_DIR, "_C_ext": os.path.join(HIP_DIR, "ext"),
              "_C_hybrid": os.path.join(HIP_DIR, "hybrid"),
              "_C_gated": os.path.join(HIP_DIR, "gated"),
              "_C_routed": os.path.join(HIP_DIR, "routed")}
only = [n for n in os.environ.get("HELIX_BUILD_ONLY", "").split(",") if n]

setup(
    name="helix_amd_C",
    ext_modules=[extension(n, d) for n, d in EXTENSIONS.items()
                 if not only or n in only],
    cmdclass={"build_ext": BuildExtension},
)
