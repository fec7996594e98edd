"""In-tree build of the gfx950 HIP extensions.

    PYTORCH_ROCM_ARCH=gfx950 python setup.py build_ext --inplace

The .so files land next to the package (aurora_amd/_hip_*.so); no JIT cache
involved. AURORA_EXTENSIONS=_hip_ops builds only what the decoders need.
"""
import os

os.environ.setdefault("PYTORCH_ROCM_ARCH", "gfx950")

from setuptools import setup
from torch.utils.cpp_extension import BuildExtension, CUDAExtension

CSRC = "aurora_amd/ops/csrc/"
EXTENSIONS = {
    # decoder kernels
    "_hip_ops": ["bindings.cpp", "elementwise.hip", "attention_decode.hip",
                 "attention_prefill.hip", "skinny_gemm.hip", "residual_norm.hip",
                 "attention_rows.hip", "recurrence.hip", "moe.hip", "sublayer.hip",
                 "latent_attention.hip", "output_norm.hip", "conv_heads.hip"],
    # sentence encoder, vector search, one-shot all-reduce
    "_hip_aux": ["bindings_aux.cpp", "encoder.hip", "allreduce.hip"],
}
wanted = os.environ.get("AURORA_EXTENSIONS", "").split(",")
names = [n for n in EXTENSIONS if n in wanted] or list(EXTENSIONS)

setup(
    name="aurora_amd_hip_ops",
    ext_modules=[
        CUDAExtension(
            name=f"aurora_amd.{name}",
            sources=[CSRC + f for f in EXTENSIONS[name]],
            extra_compile_args={
                "cxx": ["-O3", "-std=c++17"],
                # no packed fp32 instructions: some of their forms have given
                # wrong results on this hardware
                "nvcc": ["-O3", "-std=c++17", "--offload-arch=gfx950",
                         "-Xclang", "-target-feature",
                         "-Xclang", "-packed-fp32-ops"],
            },
        )
        for name in names
    ],
    cmdclass={"build_ext": BuildExtension.with_options(no_python_abi_suffix=False)},
)
