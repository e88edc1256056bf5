"""In-tree build of the native extensions for MI355X (gfx950).

    PYTORCH_ROCM_ARCH=gfx950 python setup.py build_ext --inplace

The built .so lands inside quickstart_streaming_agents_amd/ so the gpurun
snapshot carries it (it is git-ignored; history stays source-only).
hipcc cross-compiles gfx950 without a GPU present.
"""

import os

from setuptools import setup

os.environ.setdefault("PYTORCH_ROCM_ARCH", "gfx950")

from torch.utils.cpp_extension import BuildExtension, CUDAExtension  # noqa: E402

ROOT = os.path.dirname(os.path.abspath(__file__))
HIP_DIR = os.path.join(ROOT, "quickstart_streaming_agents_amd", "ops", "hip")

# Packed f32 vector instructions stay off: the compiler forms them from plain
# float code, and some of their forms are not reliable on this hardware.
HIP_FLAGS = ["-O3", "-std=c++17", "--offload-arch=gfx950",
             "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]

# module -> sources.  qsa_hip: streaming operators, retrieval, the Llama /
# Mixtral / encoder kernels.  qsa_lm_hip: the mixer decoders' kernels; it
# builds alone in well under a minute when that is all a program needs
# (QSA_BUILD=qsa_lm_hip).
MODULES = {
    "qsa_hip": ["ops.cpp", "avro_codec.cpp", "elementwise.hip",
                "paged_attn.hip", "skinny_gemm.hip", "skinny_gemm_fp8.hip",
                "hash_join.hip", "gemm_fp8_batch.hip", "topk_cosine.hip",
                "streaming.hip"],
    "qsa_lm_hip": ["lm_ops.cpp", "lm_elementwise.hip", "retention.hip",
                   "latent_attn.hip", "skinny_gemm.hip"],
}
wanted = os.environ.get("QSA_BUILD", ",".join(MODULES)).split(",")

from setuptools import find_packages  # noqa: E402

setup(
    name="quickstart-streaming-agents-amd",
    version="0.1.0",
    description=("MI355X-native streaming-agent engine: Kafka-wire "
                 "ingest, Flink-SQL-subset CREATE AGENT surface, "
                 "hand-written CDNA4 HIP kernels, RCCL over xGMI"),
    packages=find_packages(include=["quickstart_streaming_agents_amd*"]),
    package_data={"quickstart_streaming_agents_amd": [
        "labs/sql/*.sql", "data/*.csv", "data/*.json"]},
    python_requires=">=3.10",
    entry_points={"console_scripts": [
        "qsa=quickstart_streaming_agents_amd.cli:main"]},
    ext_modules=[
        CUDAExtension(
            name=f"quickstart_streaming_agents_amd.{mod}",
            sources=[os.path.join(HIP_DIR, f) for f in MODULES[mod]],
            extra_compile_args={"cxx": ["-O3", "-std=c++17"],
                                "nvcc": HIP_FLAGS},
        ) for mod in wanted
    ],
    cmdclass={"build_ext": BuildExtension.with_options(use_ninja=True)},
)
