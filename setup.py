"""In-tree build of the native components.

Two extensions, built with `python setup.py build_ext --inplace` so the .so
files live inside the package and travel with the repo snapshot:
  * llm_d_inference_scheduler_amd._router_core  — C++ router core (pybind11,
    CPU): prefix index + chained hashing, scheduler hot loop, flow queues.
  * llm_d_inference_scheduler_amd._hip_ops      — gfx950 HIP kernels (torch
    extension, hipcc --offload-arch=gfx950): prefix hash/match, paged KV,
    fused norm/rope/act, GQA decode attention.
  * llm_d_inference_scheduler_amd._hip_layered  — gfx950 HIP kernels of the
    layer-listed designs (delta rule, latent and grouped attention,
    experts, 32-bit stream).

LDS_AMD_ONLY=name,... builds only the named modules (e.g. _hip_layered).
"""
import os
import sys

from setuptools import setup

os.environ.setdefault("PYTORCH_ROCM_ARCH", "gfx950")

from pybind11.setup_helpers import Pybind11Extension
from torch.utils import cpp_extension

ROOT = os.path.dirname(os.path.abspath(__file__))

router_core = Pybind11Extension(
    "llm_d_inference_scheduler_amd._router_core",
    sources=["csrc/router/bindings.cpp"],
    cxx_std=17,
    extra_compile_args=["-O3"],
)

HIP_ARGS = {
    "cxx": ["-O3"],
    # packed fp32 instructions stay off: some of their forms have given wrong
    # results on this hardware
    "nvcc": ["-O3", "--offload-arch=gfx950", "-std=c++17",
             "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"],
}

hip_ops = cpp_extension.CUDAExtension(
    name="llm_d_inference_scheduler_amd._hip_ops",
    sources=[
        "csrc/hip/ops.hip",
        "csrc/hip/prefix_kernels.hip",
        "csrc/hip/norm_rope_act.hip",
        "csrc/hip/kv_cache.hip",
        "csrc/hip/paged_attention.hip",
        "csrc/hip/flash_prefill.hip",
        "csrc/hip/flash_prefill_glds.hip",
    ],
    extra_compile_args=HIP_ARGS,
)

hip_layered = cpp_extension.CUDAExtension(
    name="llm_d_inference_scheduler_amd._hip_layered",
    sources=[
        "csrc/hip/layered/ops.hip",
        "csrc/hip/layered/residual_norm.hip",
        "csrc/hip/layered/delta_rule.hip",
        "csrc/hip/layered/delta_chunk.hip",
        "csrc/hip/layered/attention.hip",
        "csrc/hip/layered/paged_decode.hip",
        "csrc/hip/layered/context_prefill.hip",
        "csrc/hip/layered/experts.hip",
        "csrc/hip/layered/ops_grouped.hip",
    ],
    extra_compile_args=HIP_ARGS,
)

ext_modules = [router_core]
if os.environ.get("LDS_AMD_SKIP_HIP", "0") != "1":
    ext_modules += [hip_ops, hip_layered]
only = os.environ.get("LDS_AMD_ONLY", "")
if only:
    ext_modules = [e for e in ext_modules
                   if e.name.rsplit(".", 1)[-1] in only.split(",")]

setup(
    name="llm_d_inference_scheduler_amd",
    version="0.1.0",
    packages=["llm_d_inference_scheduler_amd"],
    ext_modules=ext_modules,
    cmdclass={"build_ext": cpp_extension.BuildExtension.with_options(use_ninja=True)},
)
