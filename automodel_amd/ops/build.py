"""In-tree build of the HIP extension (gfx950).

Compiles every ``csrc/*.hip`` + ``csrc/bind.cpp`` with hipcc in parallel and
links ``automodel_amd/ops/libamd_ops.so``. No JIT cache: the .so lives in the
package so it travels with the repo snapshot to GPU boxes.

``--decode`` links only the inference kernels (attention forward, latent and
grouped attention, linear recurrences, residual norms, decode GEMV) into ``libamd_ops_decode.so``: what a
checkout with nothing built needs to generate, in a fraction of the time.

Usage: ``python -m automodel_amd.ops.build [--force] [--decode]``
"""

from __future__ import annotations

import concurrent.futures
import hashlib
import json
import os
import subprocess
import sys

PKG_DIR = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(PKG_DIR, "csrc")
BUILD_DIR = os.path.join(PKG_DIR, "_build")
SO_PATH = os.path.join(PKG_DIR, "libamd_ops.so")
DECODE_SO_PATH = os.path.join(PKG_DIR, "libamd_ops_decode.so")
DECODE_SOURCES = ("bind_decode.cpp", "flash_attn.hip", "gemv.hip", "gqa_attn.hip",
                  "hyper.hip", "latent_attn.hip", "latent_decode.hip", "linear_scan.hip",
                  "residual_norm.hip")
ARCH = os.environ.get("PYTORCH_ROCM_ARCH", "gfx950")


def _torch_paths() -> tuple[str, str]:
    import torch

    base = os.path.dirname(torch.__file__)
    return os.path.join(base, "include"), os.path.join(base, "lib")


def _sources(decode_only: bool = False) -> list[str]:
    out = []
    for f in sorted(os.listdir(CSRC)):
        if f.endswith((".hip", ".cpp")) and (not decode_only or f in DECODE_SOURCES):
            out.append(os.path.join(CSRC, f))
    return out


def _jobs() -> int:
    return max(1, min(16, int(os.environ.get("MAX_JOBS") or os.cpu_count() or 8)))


def _hash_inputs(srcs: list[str]) -> str:
    h = hashlib.sha256()
    for f in srcs + [os.path.join(CSRC, x) for x in sorted(os.listdir(CSRC)) if x.endswith(".h")]:
        with open(f, "rb") as fh:
            h.update(fh.read())
        h.update(f.encode())
    h.update(ARCH.encode())
    return h.hexdigest()


def build(force: bool = False, verbose: bool = True, decode_only: bool = False) -> str:
    inc, lib = _torch_paths()
    srcs = _sources(decode_only)
    so_path = DECODE_SO_PATH if decode_only else SO_PATH
    stamp_path = os.path.join(BUILD_DIR, os.path.basename(so_path) + ".stamp.json")
    digest = _hash_inputs(srcs)
    if not force and os.path.exists(so_path) and os.path.exists(stamp_path):
        try:
            if json.load(open(stamp_path)).get("digest") == digest:
                if verbose:
                    print(f"[amd_ops] up to date: {so_path}")
                return so_path
        except Exception:
            pass

    os.makedirs(BUILD_DIR, exist_ok=True)
    cflags = [
        f"--offload-arch={ARCH}", "-O3", "-std=c++17", "-fPIC",
        f"-I{inc}", f"-I{os.path.join(inc, 'torch/csrc/api/include')}",
        "-D_GLIBCXX_USE_CXX11_ABI=1", "-DUSE_ROCM", "-D__HIP_PLATFORM_AMD__",
        "-Wno-unused-result",
        # no v_pk_{add,mul,fma}_f32: some packed-f32 forms have returned wrong
        # results on this hardware (the host pass warns about the feature name)
        "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    ]

    def compile_one(src: str) -> str:
        obj = os.path.join(BUILD_DIR, os.path.basename(src) + ".o")
        cmd = ["hipcc", *cflags, "-c", src, "-o", obj]
        if verbose:
            print(f"[amd_ops] hipcc -c {os.path.basename(src)}")
        r = subprocess.run(cmd, capture_output=True, text=True)
        if r.returncode != 0:
            raise RuntimeError(f"hipcc failed for {src}:\n{r.stdout}\n{r.stderr}")
        return obj

    with concurrent.futures.ThreadPoolExecutor(max_workers=min(_jobs(), len(srcs))) as ex:
        objs = list(ex.map(compile_one, srcs))

    tmp_so = f"{so_path}.{os.getpid()}.tmp"    # a reader never sees half a library
    link = [
        "hipcc", f"--offload-arch={ARCH}", "-shared", "-fPIC", *objs,
        f"-L{lib}", "-ltorch", "-ltorch_hip", "-ltorch_cpu", "-lc10", "-lc10_hip",
        "-lamdhip64", f"-Wl,-rpath,{lib}", "-o", tmp_so,
    ]
    if verbose:
        print(f"[amd_ops] linking {os.path.basename(so_path)}")
    r = subprocess.run(link, capture_output=True, text=True)
    if r.returncode != 0:
        raise RuntimeError(f"link failed:\n{r.stdout}\n{r.stderr}")
    os.replace(tmp_so, so_path)
    with open(stamp_path, "w") as f:
        json.dump({"digest": digest}, f)
    if verbose:
        print(f"[amd_ops] built {so_path}")
    return so_path


if __name__ == "__main__":
    build(force="--force" in sys.argv, decode_only="--decode" in sys.argv)
