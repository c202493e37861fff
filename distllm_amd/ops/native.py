"""The compiled HIP extensions, loaded once and seen as one namespace.

The kernels are built as a few extension modules (see setup.py); callers
look an op up here by name and do not care which module holds it. A
module that is not built raises where one of its ops is used, so a
process can run with only the modules that its model needs.
"""

from __future__ import annotations

import importlib

EXTENSIONS = ("_hip_gemm", "_hip_residual", "_hip_latent", "_hip_hybrid",
              "_hip_chunked", "_hip_experts", "_hip_lru", "_hip_retention",
              "_hip_ops")


class Native:
    """Attribute access resolves over every extension that is built."""

    def __init__(self):
        self.modules: dict[str, object] = {}
        self.errors: dict[str, Exception] = {}
        for name in EXTENSIONS:
            try:
                self.modules[name] = importlib.import_module(
                    f"distllm_amd.ops.{name}")
            except Exception as e:  # not built, or built elsewhere
                self.errors[name] = e

    def require(self, name: str) -> None:
        if name not in self.modules:
            raise RuntimeError(
                f"distllm_amd HIP extension {name} is not built but a GPU "
                "tensor reached the ops layer. Build with "
                "`python setup.py build_ext --inplace` (PYTORCH_ROCM_ARCH="
                f"gfx950). Import error: {self.errors.get(name)!r}"
            )

    def __getattr__(self, op: str):
        for mod in self.__dict__.get("modules", {}).values():
            if hasattr(mod, op):
                return getattr(mod, op)
        raise AttributeError(
            f"no HIP op {op!r} in {sorted(self.__dict__['modules'])}; "
            f"not loaded: {self.__dict__['errors']!r}")
