"""Compile HIP extensions on first use in a checkout that has none.

Imports neither torch nor the ops package, so it can run before them.
"""

from __future__ import annotations

import json
import os
import subprocess
import sys
from pathlib import Path

ROOT = Path(__file__).resolve().parents[1]


# config.json "architecture" -> the extensions that the model's steps use
NEEDED = {"Kanotar": ("_hip_gemm", "_hip_residual", "_hip_latent"),
          "Bufulorn": ("_hip_gemm", "_hip_residual", "_hip_hybrid",
                       "_hip_chunked", "_hip_experts"),
          "Tebasun": ("_hip_gemm", "_hip_residual", "_hip_hybrid",
                      "_hip_lru"),
          "Kedelorn": ("_hip_gemm", "_hip_residual", "_hip_latent",
                       "_hip_experts", "_hip_retention")}


def needed_for(model_dir: str) -> tuple[str, ...]:
    """Extensions for a checkpoint folder; none if it names no
    architecture that is described in full."""
    f = Path(model_dir) / "config.json"
    if not f.is_file():
        return ()
    return NEEDED.get(json.loads(f.read_text()).get("architecture"), ())


def is_built(name: str) -> bool:
    return any((ROOT / "distllm_amd" / "ops").glob(f"{name}.*.so"))


def ensure_built(*names: str) -> None:
    """Build the named extension modules (setup.py lists them) that have
    no library in the tree yet, and no others."""
    missing = [n for n in names if not is_built(n)]
    if not missing:
        return
    env = dict(os.environ, PYTORCH_ROCM_ARCH="gfx950",
               DISTLLM_EXT=",".join(missing))
    subprocess.run(
        [sys.executable, "setup.py", "build_ext", "--inplace"],
        cwd=ROOT, env=env, check=True, stdout=sys.stderr,
    )
