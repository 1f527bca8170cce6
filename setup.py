"""In-tree build of the gfx950 HIP extensions.

    PYTORCH_ROCM_ARCH=gfx950 python setup.py build_ext --inplace

  lfmq_hip  weight-quantized Llama / Mixtral / OPT kernels
  lfmq_seq  recurrent, attention and expert layers on packed batches, and
            the small ops that every model uses

LFMQ_EXTENSIONS=lfmq_seq builds only the named ones (comma-separated).
The built .so files land at the repo root, next to the package.
"""
import os

from setuptools import setup
from torch.utils.cpp_extension import BuildExtension, CUDAExtension

os.environ.setdefault("PYTORCH_ROCM_ARCH", "gfx950")

# LFMQ_ASAN=1: address-sanitized build of the HOST side of the extension
# (binding/launch logic).  Run with
# LD_PRELOAD=$(clang -print-file-name=libclang_rt.asan-x86_64.so).
_ASAN = os.environ.get("LFMQ_ASAN", "0") == "1"
_CXX_FLAGS = ["-O3", "-std=c++17"] + (
    ["-fsanitize=address", "-fno-omit-frame-pointer"] if _ASAN else [])

SOURCES = [
    "csrc/ext.hip",
    "csrc/pack.hip",
    "csrc/rmsnorm.hip",
    "csrc/rope.hip",
    "csrc/elementwise.hip",
    "csrc/dq_gemv.hip",
    "csrc/dq_gemv_mfma.hip",
    "csrc/dq_gemm.hip",
    "csrc/hessian.hip",
    "csrc/attn_decode.hip",
    "csrc/attn_prefill.hip",
    "csrc/qkv_rope_append.hip",
    "csrc/sample.hip",
    "csrc/probe.hip",
    "csrc/grouped_dq_gemm.hip",
    "csrc/engine.hip",
    "csrc/moe_route.hip",
]

SEQ_SOURCES = [
    "csrc/seq_ext.hip",
    "csrc/bigram_embed.hip",
    "csrc/fused_norm.hip",
    "csrc/mlstm.hip",
    "csrc/mlstm_chunk.hip",
    "csrc/latent_prep.hip",
    "csrc/attn_window.hip",
    "csrc/attn_window_mfma.hip",
    "csrc/attn_latent_mfma.hip",
    "csrc/attn_grouped_decode.hip",
    "csrc/qk_prep.hip",
    "csrc/gated_lru.hip",
    "csrc/moe_experts.hip",
    "csrc/post_norm.hip",
    "csrc/elementwise.hip",
    "csrc/sample.hip",
]

# packed fp32 instructions off: some of their forms have returned wrong
# results on this hardware
_HIP_FLAGS = ["-O3", "-std=c++17", "-Xclang", "-target-feature",
              "-Xclang", "-packed-fp32-ops"]

_ALL = {"lfmq_hip": SOURCES, "lfmq_seq": SEQ_SOURCES}
_WANT = [n for n in os.environ.get("LFMQ_EXTENSIONS", "").split(",") if n]
for _n in _WANT:
    if _n not in _ALL:
        raise SystemExit(f"LFMQ_EXTENSIONS: unknown extension {_n!r}")

setup(
    name="lfmq_hip",
    ext_modules=[
        CUDAExtension(
            name=name,
            sources=sources,
            extra_compile_args={"cxx": _CXX_FLAGS, "nvcc": _HIP_FLAGS},
        )
        for name, sources in _ALL.items() if not _WANT or name in _WANT
    ],
    cmdclass={"build_ext": BuildExtension.with_options(use_ninja=True)},
)
