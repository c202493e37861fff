"""Build the distllm-amd HIP extensions in-tree for gfx950 (MI355X).

    python setup.py build_ext --inplace

The kernels are grouped into a few extensions, so that a process which
needs one group does not have to compile the others:

    _hip_gemm      matrix products and gated units (every model)
    _hip_residual  boundaries of fp32 residual streams, rotation tables
    _hip_latent    latent attention
    _hip_hybrid    attention over pages of keys and values, delta rules
    _hip_chunked   the same attention with capped scores, chunk by chunk
    _hip_experts   xIELU, routed experts
    _hip_lru       linear recurrent unit
    _hip_retention retention
    _hip_ops       everything else

DISTLLM_EXT=_hip_gemm,_hip_latent restricts a build to the named ones.
The resulting distllm_amd/ops/_hip_*.so are git-ignored.
"""

import os
from pathlib import Path

os.environ.setdefault("PYTORCH_ROCM_ARCH", "gfx950")

from setuptools import setup
from torch.utils.cpp_extension import BuildExtension, CUDAExtension

CSRC = Path(__file__).parent / "distllm_amd" / "ops" / "csrc"
GROUPS = {
    "_hip_gemm": ["ext_gemm.cpp", "blt_gemm.cpp", "gemm.hip", "gemm8.hip",
                  "gemm16.hip", "decode_gemm.hip", "clamped_glu.hip",
                  "gelu_rows.hip", "relu2.hip"],
    "_hip_latent": ["ext_latent.cpp", "latent_attention.hip",
                    "latent_decode.hip", "window_attention.hip"],
    "_hip_residual": ["ext_residual.cpp", "residual_norms.hip", "streams.hip",
                      "rotation.hip"],
    "_hip_hybrid": ["ext_hybrid.cpp", "chunk_attention.hip",
                    "sink_rows.hip", "sink_flash.hip", "delta_rule.hip",
                    "delta_chunk.hip", "delta_channel.hip"],
    "_hip_chunked": ["ext_chunked.cpp", "chunk_rows.hip", "chunk_flash.hip"],
    "_hip_experts": ["ext_experts.cpp", "experts.hip", "expert_gemm16.hip",
                     "xielu.hip"],
    "_hip_lru": ["ext_lru.cpp", "lru.hip"],
    "_hip_retention": ["ext_retention.cpp", "retention.hip"],
}
_taken = {s for group in GROUPS.values() for s in group}
# *_hip.hip files are torch-hipify build artifacts — exclude them.
GROUPS["_hip_ops"] = ["ext.cpp"] + sorted(
    p.name for p in CSRC.glob("*.hip")
    if not p.name.endswith("_hip.hip") and p.name not in _taken
)

wanted = os.environ.get("DISTLLM_EXT", "")
names = [n for n in wanted.split(",") if n] or list(GROUPS)

# hipcc -O3 forms packed-FP32 instructions from ordinary float code; some
# of their forms have given wrong results on this hardware, so the
# feature is off for every kernel.
HIPCC_FLAGS = ["-O3", "--offload-arch=gfx950", "-std=c++17",
               "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]

setup(
    name="distllm_amd_ops",
    ext_modules=[
        CUDAExtension(
            name=f"distllm_amd.ops.{name}",
            sources=[str(CSRC / s) for s in GROUPS[name]],
            extra_compile_args={"cxx": ["-O3"], "nvcc": HIPCC_FLAGS},
            libraries=["hipblaslt"] if name == "_hip_gemm" else [],
        )
        for name in names
    ],
    cmdclass={"build_ext": BuildExtension},
)
