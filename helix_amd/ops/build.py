"""In-tree build of the native extensions, on demand.

A source checkout has no built libraries; a program that needs one calls
ensure() before it imports helix_amd.ops. Only the named extensions are
compiled (gfx950, cross-compilation needs no GPU).
"""
from __future__ import annotations

import glob
import importlib
import os
import subprocess
import sys

ROOT = os.path.dirname(os.path.dirname(os.path.dirname(
    os.path.abspath(__file__))))


def is_built(name: str) -> bool:
    return bool(glob.glob(os.path.join(ROOT, "helix_amd", f"{name}.*.so")))


def ensure(names: str) -> None:
    """Compile the extensions (names with commas between them) whose library
    is not there. The compiler's output goes to standard error."""
    names = ",".join(n for n in names.split(",") if not is_built(n))
    if not names:
        return
    env = dict(os.environ, PYTORCH_ROCM_ARCH="gfx950", HELIX_BUILD_ONLY=names)
    subprocess.run([sys.executable, "setup.py", "build_ext", "--inplace"],
                   cwd=ROOT, env=env, check=True, stdout=sys.stderr)


_loaded: dict = {}


def load(name: str):
    """Extension `name`, imported at first use (a program may build it after
    helix_amd.ops was imported)."""
    if name not in _loaded:
        try:
            _loaded[name] = importlib.import_module(f"helix_amd.{name}")
        except ImportError as e:
            raise RuntimeError(
                f"helix_amd.{name} native extension is not built but a GPU "
                "tensor was passed. Build it with `python setup.py build_ext "
                "--inplace` (PYTORCH_ROCM_ARCH=gfx950). Import error: "
                f"{e}") from e
    return _loaded[name]
