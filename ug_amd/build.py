"""Build recipe for the native libraries (run on the CPU box; hipcc cross-compiles gfx950).

    python -m ug_amd.build            # libughip.so + libug_host.so (+ the oracle's test library)

libughip.so   the backend behind the C ABI of include/ughip.h (HIP kernels, hiprtc lowering)
libug_host.so host-side front-end (lazy buffer graph, scheduler, llama) over that C ABI
oracle/_build/libug_oracle.so   CPU restatement of ug's CPU backend -- test infrastructure only
"""
import os
import subprocess
import sys

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
CSRC = os.path.join(ROOT, "ug_amd", "csrc")
LIB = os.path.join(ROOT, "ug_amd", "lib")
INC = os.path.join(ROOT, "include")
ROCM = os.environ.get("ROCM_PATH", "/opt/rocm")

# -packed-fp32-ops is switched off on purpose: packed f32 forms have produced wrong results on
# this hardware pool; hipcc's host pass does not know the feature and warns (harmless).
HIP_FLAGS = ["--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
             "-Wno-unused-value", "-Wno-unused-command-line-argument"]


def _run(cmd):
    print("+", " ".join(cmd), flush=True)
    p = subprocess.run(cmd, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)
    out = "\n".join(l for l in p.stdout.splitlines() if "packed-fp32-ops" not in l and l.strip())
    if out:
        print(out, flush=True)
    if p.returncode != 0:
        raise RuntimeError("build step failed: " + " ".join(cmd))


UGHIP_SOURCES = ("runtime.cpp", "lower_hip.cpp", "llama_ops.hip", "matmul.hip", "gemm_tiled.hip", "gemm_dma.hip", "gemm_dma_f32.hip", "rows_x3.hip", "attention.hip", "fused_linear.hip", "convert.hip",
                 "rows_product.hip", "row_step.hip", "row_norms.hip", "latent_attention.hip", "grouped_attention.hip", "ssm.hip", "delta.hip", "moe.hip")


def build_ughip(only_changed=False):
    """One object per source file, compiled side by side, then one link.  only_changed (a developer's
    shortcut, `python -m ug_amd.build ughip-changed`): keep objects newer than their source and every header."""
    from concurrent.futures import ThreadPoolExecutor
    os.makedirs(LIB, exist_ok=True)
    src = os.path.join(CSRC, "ughip")
    obj_dir = os.path.join(LIB, "obj")
    os.makedirs(obj_dir, exist_ok=True)
    hipcc = os.path.join(ROCM, "bin", "hipcc")
    headers = [os.path.join(src, f) for f in os.listdir(src) if f.endswith(".h")] + [os.path.join(INC, f) for f in os.listdir(INC)]
    newest_header = max(os.path.getmtime(h) for h in headers)
    jobs, objs = [], []
    for f in UGHIP_SOURCES:
        o = os.path.join(obj_dir, f.rsplit(".", 1)[0] + ".o")
        objs.append(o)
        path = os.path.join(src, f)
        if only_changed and os.path.exists(o) and os.path.getmtime(o) > max(os.path.getmtime(path), newest_header):
            continue
        jobs.append([hipcc] + HIP_FLAGS + ["-c", "-I" + INC, "-I" + src, path, "-o", o])
    with ThreadPoolExecutor(max_workers=min(8, max(1, len(jobs)))) as pool:
        list(pool.map(_run, jobs))
    _run([hipcc, "--offload-arch=gfx950", "-shared", "-fPIC"] + objs +
         ["-L" + os.path.join(ROCM, "lib"), "-lhiprtc", "-Wl,-rpath," + os.path.join(ROCM, "lib"), "-o", os.path.join(LIB, "libughip.so")])


def build_host():
    src = os.path.join(CSRC, "host")
    files = [os.path.join(src, f) for f in ("ug/lower_op.cpp", "ug/lazy_buffer.cpp", "ug/schedule.cpp", "ug/safetensors.cpp", "hip_device.cpp", "llama.cpp", "hybrid_ops.cpp", "hybrid.cpp", "grouped_attention.cpp", "channel_delta.cpp", "decoder.cpp", "capi.cpp")]
    _run(["g++", "-std=c++17", "-O2", "-fPIC", "-shared", "-Wall", "-I" + INC, "-I" + src] + files +
         ["-L" + LIB, "-lughip", "-Wl,-rpath,$ORIGIN", "-lpthread", "-o", os.path.join(LIB, "libug_host.so")])


def build_oracle():
    mk = os.path.join(ROOT, "oracle", "Makefile")
    if os.path.exists(mk):
        _run(["make", "-s", "-C", os.path.join(ROOT, "oracle")])


def ensure_built():
    """Builds what a model needs to run (the two product libraries) where they are missing, e.g. in a fresh checkout."""
    if not all(os.path.exists(os.path.join(LIB, f)) for f in ("libughip.so", "libug_host.so")):
        build_ughip()
        build_host()


def build_all():
    build_ughip()
    build_host()
    build_oracle()


if __name__ == "__main__":
    what = sys.argv[1:] or ["all"]
    for w in what:
        {"all": build_all, "ughip": build_ughip, "ughip-changed": lambda: build_ughip(True), "host": build_host, "oracle": build_oracle}[w]()
