"""Build recipe for the HIP library (gfx950 only).

    python ornith-rs_amd/build.py          # compile csrc/*.hip, *.cpp -> libornith_hip.so
    python ornith-rs_amd/build.py Pigodra  # only what models of that design need -> build/libornith_Pigodra.so

hipcc cross-compiles without a GPU. Every translation unit is compiled with
-ffp-contract=off (the only fused multiply-adds are the explicit ones, so results
do not depend on what the optimiser chooses to contract), with packed-fp32
instruction selection disabled, and with kernel-argument preloading on.
"""
import concurrent.futures
import os
import shutil
import subprocess
import sys

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
OBJ = os.path.join(HERE, "build")
LIB = os.path.join(HERE, "libornith_hip.so")

HIPCC = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"
FLAGS = [
    "--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-ffp-contract=off",
    "-fno-fast-math", "-fvisibility=hidden", "-Wall", "-Wno-unused-function",
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    # the first 14 dwords of a kernel's flat (non-struct) arguments arrive in scalar registers
    # with the wavefront instead of through a scalar load (gfx950 kernel-argument preloading)
    "-mllvm", "-amdgpu-kernarg-preload-count=14",
    "-Wno-unknown-warning-option", "-Wno-unused-command-line-argument", "-Wno-pass-failed",
]


# extra compiler flags for one-off builds (e.g. -DORN_TIMING: per-workgroup time stamps)
FLAGS += os.environ.get("ORN_EXTRA_FLAGS", "").split()


# What every design needs, and what each design of the registry adds (a design that is not listed
# needs the whole library).
CORE = ["runtime.hip", "weights.cpp", "safetensors.cpp", "model.cpp", "rope.cpp", "engine.cpp", "sample.hip", "sampler.hip"]
DESIGNS = {
    "Pigodra": ["pigodra.cpp", "stack.cpp", "dense_rows.hip", "mix_mlstm.cpp", "mlstm.hip", "mix_diff_attn.cpp", "diff_attn.hip"],
    "Ranavik": ["ranavik.cpp", "stack.cpp", "dense_rows.hip", "mix_retention.cpp", "retention.hip", "mix_latent_attn.cpp",
                "latent_attn.hip"],
}


def sources(design=None):
    if design is not None:
        return CORE + DESIGNS[design]
    return sorted(f for f in os.listdir(CSRC) if f.endswith((".hip", ".cpp")))


def library(design=None):
    return LIB if design is None else os.path.join(OBJ, f"libornith_{design}.so")


def _compile(src):
    obj = os.path.join(OBJ, os.path.splitext(src)[0] + ".o")
    cmd = [HIPCC, *FLAGS, "-x", "hip", "-c", os.path.join(CSRC, src), "-o", obj]
    r = subprocess.run(cmd, capture_output=True, text=True)
    # hipcc's host pass does not know the packed-fp32 feature and says so; drop that line
    err = "\n".join(l for l in r.stderr.splitlines() if "packed-fp32-ops" not in l)
    return src, obj, r.returncode, err


def build(verbose=True, jobs=8, design=None):
    os.makedirs(OBJ, exist_ok=True)
    objs = []
    with concurrent.futures.ThreadPoolExecutor(max_workers=jobs) as ex:
        for src, obj, rc, err in ex.map(_compile, sources(design)):
            if verbose and err.strip():
                print(f"[{src}]\n{err}", file=sys.stderr)
            if rc != 0:
                raise RuntimeError(f"hipcc failed on {src}")
            objs.append(obj)
    # linked beside its place and moved there whole, so that nobody loads half a library
    out = library(design)
    part = f"{out}.{os.getpid()}"
    cmd = [HIPCC, "--offload-arch=gfx950", "-shared", "-fPIC", "-Wl,-z,defs", "-o", part, *objs]
    r = subprocess.run(cmd, capture_output=True, text=True)
    if r.returncode != 0:
        print(r.stderr, file=sys.stderr)
        raise RuntimeError("link failed")
    os.replace(part, out)
    return out


def ensure(design=None):
    """The path of a library that serves `design`: the whole one if it is there, else one of the
    design's own parts, compiled if it is missing or older than its sources (one process at a time)."""
    import fcntl
    if design not in DESIGNS:
        design = None
    if os.path.exists(LIB):
        return LIB
    os.makedirs(OBJ, exist_ok=True)
    with open(os.path.join(OBJ, ".lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        path = library(design)
        newest = max(os.path.getmtime(os.path.join(CSRC, f)) for f in os.listdir(CSRC))
        return path if os.path.exists(path) and os.path.getmtime(path) >= newest else build(verbose=False, design=design)


if __name__ == "__main__":
    print(build(design=sys.argv[1] if len(sys.argv) > 1 else None))
