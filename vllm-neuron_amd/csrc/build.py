#!/usr/bin/env python3
"""Build libmi355x_vllm.so for gfx950 with hipcc (cross-compiles without a GPU).

    python vllm-neuron_amd/csrc/build.py [--force | --if-missing]

Objects go to csrc/build/, the library next to the sources (in-tree, git-ignored: it
travels to the GPU box with the snapshot).
"""
import concurrent.futures as cf
import os
import shutil
import subprocess
import sys

HERE = os.path.dirname(os.path.abspath(__file__))
HIPCC = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"
SOURCES = ["gemv_bf16.hip", "gemv_f8.hip", "gemv_i8.hip", "linear_kernels.hip", "attn_kernels.hip", "misc_kernels.hip", "stack_kernels.hip",
           "window_attn.hip", "latent_attn.hip", "delta_rule.hip", "ssm.hip", "experts.hip", "stack.hip", "stack_ops.hip", "model.hip", "tp_group.hip"]
HEADERS = ["mi_common.h", "linear_device.h", "linear_kernels.h", "attn_kernels.h", "misc_kernels.h", "model_internal.h", "stack_kernels.h", "window_attn.h", "latent_attn.h", "delta_rule.h", "ssm.h", "experts.h", "stack.h", "tp_group.h",
           os.path.join("..", "..", "include", "mi355x_vllm.h")]
LIB = os.path.join(HERE, "libmi355x_vllm.so")
FLAGS = ["--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-Wall", "-Wno-unused-function", "-Wno-unused-value",
         "-Wno-unused-result", "-I/opt/rocm/include",
         # no packed fp32 math (v_pk_{add,mul,fma}_f32): some of its forms are not reliable on these machines
         "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]
# extra flags for probe builds (e.g. MI_EXTRA_FLAGS="-DMI_TRACE"); part of the stamp below
FLAGS += os.environ.get("MI_EXTRA_FLAGS", "").split()
STAMP = os.path.join(HERE, "build", "flags.stamp")


def _mtime(p):
    return os.path.getmtime(p) if os.path.exists(p) else 0.0


def _flags_changed():
    """An object built with other flags is stale whatever its mtime says."""
    want = " ".join(FLAGS)
    try:
        with open(STAMP) as f:
            same = f.read() == want
    except OSError:
        same = False
    if not same:
        with open(STAMP, "w") as f:
            f.write(want)
    return not same


def _compile(src, force=False):
    obj = os.path.join(HERE, "build", src.replace(".hip", ".o"))
    deps = [os.path.join(HERE, src)] + [os.path.join(HERE, h) for h in HEADERS]
    if _mtime(obj) > max(_mtime(d) for d in deps) and not force:
        return obj, ""
    cmd = [HIPCC, *FLAGS, "-c", os.path.join(HERE, src), "-o", obj]
    r = subprocess.run(cmd, capture_output=True, text=True)
    if r.returncode != 0:
        raise RuntimeError(f"hipcc failed for {src}:\n{r.stdout}\n{r.stderr}")
    return obj, r.stderr


def build(verbose=True):
    os.makedirs(os.path.join(HERE, "build"), exist_ok=True)
    force = "--force" in sys.argv or _flags_changed()
    with cf.ThreadPoolExecutor(max_workers=min(len(SOURCES), int(os.environ.get("MAX_JOBS") or os.cpu_count() or 4))) as ex:
        results = list(ex.map(lambda src: _compile(src, force), SOURCES))
    objs = [o for o, _ in results]
    for _, warn in results:
        if warn and verbose:
            sys.stderr.write(warn)
    if _mtime(LIB) < max(_mtime(o) for o in objs) or force:
        cmd = [HIPCC, "--offload-arch=gfx950", "-shared", "-fPIC", *objs, "-o", LIB,
               "-L/opt/rocm/lib", "-lrccl", "-Wl,-rpath,/opt/rocm/lib"]
        r = subprocess.run(cmd, capture_output=True, text=True)
        if r.returncode != 0:
            raise RuntimeError(f"link failed:\n{r.stdout}\n{r.stderr}")
    return LIB


if __name__ == "__main__":
    if "--if-missing" in sys.argv and os.path.exists(os.environ.get("MI355X_VLLM_LIB") or LIB):
        sys.exit(0)
    print(build())
