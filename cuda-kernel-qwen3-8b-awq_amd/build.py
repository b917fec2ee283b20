"""Compile the HIP library, the command-line programs and (optionally) the CPU oracle.

Run as a script or call build().  Everything lands in-tree next to this file
(libawq_infer.so, qwen3_awq_infer, trace_run) so that a source snapshot carries the
binaries along.

`build.py --trace-run` compiles only what replaying traces needs: the step driver, the models that are
described by a config.json and their kernels, linked into trace_run itself.
"""
import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
ROOT = os.path.dirname(HERE)
CSRC = os.path.join(HERE, "csrc")
LIB = os.path.join(HERE, "libawq_infer.so")
CLI = os.path.join(HERE, "qwen3_awq_infer")

TRACE = os.path.join(HERE, "trace_run")

# the step driver with the model registry and the operators every model uses
CORE_SOURCES = ["engine.cpp", "checkpoint.cpp", "ops.hip"]
# models described by a config.json
CONFIG_MODEL_SOURCES = ["config_model.cpp", "kugilix.cpp", "tudasun.cpp", "dense.hip", "token_ops.hip", "sublayer_ops.hip",
                        "window_attention.hip", "linear_attention.hip", "latent_attention.hip", "gated_state.hip",
                        "experts.hip"]
# the int4 model of the raw weight directory and the entry points for single kernels
INT4_SOURCES = ["gemv.hip", "gemm.hip", "prefill.hip", "attention.hip", "fused.hip", "qkv_attn.hip", "qwen3.cpp",
                "kernel_api.cpp", "layer_api.cpp", "synth.cpp"]

# -ffp-contract=off: every fma in the sources is written out; a contracted
#   a*b-c*d would break bit parity with the reference's __hmul/__hsub sequence.
# packed-fp32 ops are switched off for the whole library.
HIPCC_FLAGS = [
    "--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-fopenmp",
    "-ffp-contract=off", "-fno-fast-math", "-fhip-fp32-correctly-rounded-divide-sqrt",
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    # first 16 dwords of a kernel's arguments arrive in scalar registers at wavefront launch
    "-mllvm", "-amdgpu-kernarg-preload-count=16",
    "-Wall", "-Wno-unused-function", "-x", "hip",
]


def _run(cmd):
    res = subprocess.run(cmd, capture_output=True, text=True)
    if res.returncode != 0:
        sys.stderr.write(" ".join(cmd) + "\n" + res.stdout + res.stderr)
        raise RuntimeError("build step failed: " + cmd[0])
    return res


def _compile(sources):
    """object files of the sources, several compilers at a time"""
    hipcc = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
    objdir = os.path.join(HERE, "build")
    os.makedirs(objdir, exist_ok=True)

    def compile_one(src):
        obj = os.path.join(objdir, src + ".o")
        _run([hipcc] + HIPCC_FLAGS + ["-c", os.path.join(CSRC, src), "-o", obj])
        return obj

    with ThreadPoolExecutor(max_workers=min(8, len(sources))) as pool:
        return dict(zip(sources, pool.map(compile_one, sources)))


def _link_trace_run(objs):
    hipcc = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
    part = "%s.%d" % (TRACE, os.getpid())
    _run([hipcc, "--offload-arch=gfx950", "-fopenmp", "-o", part] +
         [objs[s] for s in ["trace_run.cpp"] + CORE_SOURCES + CONFIG_MODEL_SOURCES])
    os.replace(part, TRACE)


def build_trace_run():
    _link_trace_run(_compile(["trace_run.cpp"] + CORE_SOURCES + CONFIG_MODEL_SOURCES))
    return TRACE


def build(verbose=False, oracle=True):
    hipcc = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
    library = CORE_SOURCES + CONFIG_MODEL_SOURCES + INT4_SOURCES
    objs = _compile(library + ["trace_run.cpp"])
    _run([hipcc, "--offload-arch=gfx950", "-shared", "-fopenmp", "-o", LIB] + [objs[s] for s in library])
    _link_trace_run(objs)
    # the drop-in C++ class and the command line on top of the C ABI
    _run([hipcc, "-O2", "-std=c++17", os.path.join(CSRC, "qwen3_awq_infer.cpp"), os.path.join(CSRC, "main.cpp"),
          "-o", CLI, "-L" + HERE, "-lawq_infer", "-Wl,-rpath,$ORIGIN"])
    if oracle:
        _run(["make", "-C", os.path.join(ROOT, "oracle"), "-B"])
    if verbose:
        print("built", LIB)
    return LIB


if __name__ == "__main__":
    if sys.argv[1:] == ["--trace-run"]:
        print("built", build_trace_run())
    else:
        build(verbose=True)
