"""In-tree build of the native extensions for MI355X (gfx950).

    python setup.py build_ext --inplace

The built .so files land inside quickstart_streaming_agents_amd/ (they are
git-ignored; history stays source-only).  hipcc cross-compiles gfx950 without
a GPU present.  The sources are HIP as written: hipcc compiles them directly,
an object is rebuilt when its source, a header or this file is newer, and
QSA_FORCE=1 rebuilds everything.  QSA_BUILD=<module>[,<module>] builds only
those modules.
"""

import glob
import os
import subprocess
import sysconfig
from concurrent.futures import ThreadPoolExecutor

from setuptools import Extension, find_packages, setup
from setuptools.command.build_ext import build_ext

ROOT = os.path.dirname(os.path.abspath(__file__))
PACKAGE = "quickstart_streaming_agents_amd"
HIP_DIR = os.path.join(ROOT, PACKAGE, "ops", "hip")
ROCM = os.environ.get("ROCM_PATH", "/opt/rocm")

# Packed f32 vector instructions stay off: the compiler forms them from plain
# float code, and some of their forms are not reliable on this hardware.
HIP_FLAGS = ["-O3", "-std=c++17", "-fPIC", "--offload-arch=gfx950",
             "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]

# module -> sources.  qsa_hip: streaming operators, retrieval, the Llama /
# Mixtral / encoder kernels.  qsa_lm_hip: the mixer decoders' kernels; it
# builds alone in about a minute when that is all a program needs.
MODULES = {
    "qsa_hip": ["ops.cpp", "avro_codec.cpp", "elementwise.hip",
                "paged_attn.hip", "skinny_gemm.hip", "skinny_gemm_fp8.hip",
                "hash_join.hip", "gemm_fp8_batch.hip", "topk_cosine.hip",
                "streaming.hip"],
    "qsa_lm_hip": ["lm_ops.cpp", "lm_elementwise.hip", "retention.hip",
                   "latent_attn.hip", "short_conv.hip", "gqa_attn.hip", "ssd.hip",
                   "skinny_gemm.hip"],
}


class HipBuild(build_ext):
    """One compiler call per source, in parallel, then one link."""

    def run(self):
        from torch.utils import cpp_extension as ce
        import torch
        jobs = min(16, int(os.environ.get("MAX_JOBS") or os.cpu_count() or 8))
        inc = [f"-I{p}" for p in ce.include_paths()] + [
            f"-I{ROCM}/include", f"-I{sysconfig.get_paths()['include']}",
            f"-I{HIP_DIR}"]
        abi = int(torch._C._GLIBCXX_USE_CXX11_ABI)
        host = ["-O3", "-std=c++17", "-fPIC", "-D__HIP_PLATFORM_AMD__=1",
                "-DUSE_ROCM=1", "-DHIPBLAS_V2",
                "-DTORCH_API_INCLUDE_EXTENSION_H",
                f"-D_GLIBCXX_USE_CXX11_ABI={abi}"]
        newest = max(os.path.getmtime(p) for p in
                     glob.glob(os.path.join(HIP_DIR, "*.h")) +
                     [os.path.abspath(__file__)])
        force = self.force or os.environ.get("QSA_FORCE") == "1"

        def compile_one(job):
            mod, name = job
            src = os.path.join(HIP_DIR, name)
            obj = os.path.join(self.build_temp, mod, name + ".o")
            if not force and os.path.exists(obj) and \
                    os.path.getmtime(obj) > max(newest,
                                                os.path.getmtime(src)):
                return obj
            os.makedirs(os.path.dirname(obj), exist_ok=True)
            if name.endswith(".hip"):
                cmd = [f"{ROCM}/bin/hipcc", *HIP_FLAGS, "-c", src, "-o", obj]
            else:
                cmd = ["g++", *host, f"-DTORCH_EXTENSION_NAME={mod}", *inc,
                       "-c", src, "-o", obj]
            print(" ".join(cmd), flush=True)
            subprocess.run(cmd, check=True)
            return obj

        jobs_list = [(e.name.split(".")[-1], os.path.basename(s))
                     for e in self.extensions for s in e.sources]
        with ThreadPoolExecutor(jobs) as pool:
            objs = dict(zip(jobs_list, pool.map(compile_one, jobs_list)))
        libs = [f"-L{p}" for p in ce.library_paths()] + [
            f"-L{ROCM}/lib", "-lc10", "-ltorch", "-ltorch_cpu",
            "-ltorch_python", "-lamdhip64", "-lc10_hip", "-ltorch_hip"]
        for e in self.extensions:
            mod = e.name.split(".")[-1]
            out = self.get_ext_fullpath(e.name)
            os.makedirs(os.path.dirname(os.path.abspath(out)), exist_ok=True)
            part = out + ".part"
            subprocess.run(["g++", "-shared", "-o", part] +
                           [objs[j] for j in jobs_list if j[0] == mod] + libs,
                           check=True)
            os.replace(part, out)
            print(f"built {out}", flush=True)


wanted = os.environ.get("QSA_BUILD", ",".join(MODULES)).split(",")

setup(
    name="quickstart-streaming-agents-amd",
    version="0.1.0",
    description=("MI355X-native streaming-agent engine: Kafka-wire "
                 "ingest, Flink-SQL-subset CREATE AGENT surface, "
                 "hand-written CDNA4 HIP kernels, RCCL over xGMI"),
    packages=find_packages(include=[PACKAGE + "*"]),
    package_data={PACKAGE: ["labs/sql/*.sql", "data/*.csv", "data/*.json"]},
    python_requires=">=3.10",
    entry_points={"console_scripts": [f"qsa={PACKAGE}.cli:main"]},
    ext_modules=[
        Extension(f"{PACKAGE}.{mod}",
                  [os.path.join(HIP_DIR, f) for f in MODULES[mod]])
        for mod in wanted],
    cmdclass={"build_ext": HipBuild},
)
