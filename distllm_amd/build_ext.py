"""Compile HIP extensions on first use in a checkout that has none.

Imports neither torch nor the ops package, so it can run before them.
"""

from __future__ import annotations

import os
import subprocess
import sys
from pathlib import Path

ROOT = Path(__file__).resolve().parents[1]


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
