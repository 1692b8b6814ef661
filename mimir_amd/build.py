"""Builds libmimir_mi355x.so, the gfx950 code of this package, with hipcc.

The library is built in-tree (mimir_amd/lib/) ahead of time. `python -m
mimir_amd.build` rebuilds it; with the name of a part (PARTS) it compiles that
part's sources alone, into a library of their own with the same entry points.
ensure() does the same if nothing is built yet, for commands that are run from a
fresh checkout.
"""
from __future__ import annotations

import fcntl
import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
LIB_DIR = os.path.join(HERE, "lib")
LIB_PATH = os.path.join(LIB_DIR, "libmimir_mi355x.so")
OBJ_DIR = os.path.join(LIB_DIR, "obj")

ARCH = "gfx950"
# -packed-fp32-ops is switched off on purpose: hipcc must not form v_pk_*_f32.
DEVICE_FLAGS = ["-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]
FLAGS = ["-O3", "-std=c++17", "-fPIC", f"--offload-arch={ARCH}", "-fvisibility=hidden", "-Wall", "-Wno-unused-function",
         "-Wno-unknown-warning-option", "-ffp-contract=on"] + DEVICE_FLAGS


# Sources that make a library of their own: what the decoders of one kind need.
PARTS = {
    "stack": ("runtime", "decoder", "stack", "residual_ops", "linear_recurrence", "attention_latent", "attention_heads", "gemv_float", "gemv_bf16_rows",
              "gemm_float", "gemm_bf16", "decode_ops"),
}


def sources(part: str | None = None) -> list[str]:
    if part is not None:
        return [os.path.join(CSRC, f + ".hip") for f in PARTS[part]]
    return sorted(os.path.join(CSRC, f) for f in os.listdir(CSRC) if f.endswith(".hip"))


def lib_path(part: str | None = None) -> str:
    return LIB_PATH if part is None else os.path.join(LIB_DIR, f"libmimir_mi355x_{part}.so")


def _compile(src: str) -> str:
    obj = os.path.join(OBJ_DIR, os.path.basename(src)[:-4] + ".o")
    cmd = ["hipcc", *FLAGS, "-c", src, "-o", obj]
    r = subprocess.run(cmd, capture_output=True, text=True)
    if r.returncode != 0:
        raise RuntimeError(f"hipcc failed on {src}:\n{r.stderr[-4000:]}")
    return obj


PROBE_SRC = os.path.join(HERE, "probe", "launch_cost.hip")
PROBE_BIN = os.path.join(LIB_DIR, "launch_cost")


def build_probe() -> list[str]:
    """The stand-alone launch-cost probe (no part of the library): once as it is, once with its kernels' arguments
    preloaded into scalar registers."""
    outs = []
    for suffix, extra in (("", []), ("_preload", ["-mllvm", "-amdgpu-kernarg-preload-count=16", '-DPRELOAD_NOTE="16 SGPRs"'])):
        out = PROBE_BIN + suffix
        cmd = ["hipcc", "-O3", "-std=c++17", f"--offload-arch={ARCH}", *DEVICE_FLAGS, *extra, PROBE_SRC, "-o", out]
        r = subprocess.run(cmd, capture_output=True, text=True)
        if r.returncode != 0:
            raise RuntimeError(f"hipcc failed on {PROBE_SRC}:\n{r.stderr[-4000:]}")
        outs.append(out)
    return outs


def build(verbose: bool = False, part: str | None = None) -> str:
    """Compiles every .hip source (or a part's) for gfx950 and links the shared library."""
    os.makedirs(OBJ_DIR, exist_ok=True)
    srcs = sources(part)
    with ThreadPoolExecutor(max_workers=min(8, len(srcs))) as ex:
        objs = list(ex.map(_compile, srcs))
    out = lib_path(part)
    tmp = out + ".tmp"
    cmd = ["hipcc", "-shared", "-fPIC", f"--offload-arch={ARCH}", "-o", tmp, *objs]
    if part is not None:  # a reference into another part's sources shows here and not when the library is loaded
        cmd.append("-Wl,-z,defs")
    r = subprocess.run(cmd, capture_output=True, text=True)
    if r.returncode != 0:
        raise RuntimeError(f"link failed:\n{r.stderr[-4000:]}")
    os.replace(tmp, out)
    if part is None:
        build_probe()
    if verbose:
        print(f"built {out} from {len(srcs)} sources", file=sys.stderr)
    return out


def ensure(part: str | None = None) -> None:
    """Builds the library, or the part of it that is asked for, if neither is there. One process builds at a time."""
    def there():
        return os.path.exists(LIB_PATH) or (part is not None and os.path.exists(lib_path(part)))
    if there():
        return
    os.makedirs(LIB_DIR, exist_ok=True)
    with open(os.path.join(LIB_DIR, "build.lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if not there():
            build(part=part)


if __name__ == "__main__":
    build(verbose=True, part=sys.argv[1] if len(sys.argv) > 1 else None)
