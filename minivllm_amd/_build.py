"""Builds libminivllm_amd.so (gfx950) in-tree with hipcc.

``python -m minivllm_amd._build`` or ``build_library()``.  The library is
written next to the sources' package (minivllm_amd/libminivllm_amd.so).

``ensure_library(sources)`` is for programs that start in a checkout without a built library and need a few kernel
families only: it uses the full library if there is one and otherwise builds (once) a partial library of those sources.
"""
from __future__ import annotations

import hashlib
import os
import shutil
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

PKG_DIR = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(PKG_DIR, "csrc")
LIB_PATH = os.path.join(PKG_DIR, "libminivllm_amd.so")
PROBE_LIB_PATH = os.path.join(PKG_DIR, "libmvllm_probe.so")      # measurement support for bench.py, not an operator
PROBE_SOURCES = ["mfma_probe.hip"]
SOURCES = ["capi.hip", "store_kvcache.hip", "paged_decode.hip", "prefill_varlen.hip", "prefill_other_dims.hip", "prefill_half_step_dims.hip", "prefill_pingpong.hip", "prefill_staged.hip", "prefill_split.hip", "prefill_f32.hip", "qk_norm_rope_store.hip", "sampler.hip",
           "rms_norm.hip", "activation.hip", "linear_small.hip", "norm_conv.hip", "head_rope.hip", "gate_linear.hip", "mlstm.hip", "mlstm_chunk.hip",
           "decay_memory.hip", "latent.hip", "moe.hip", "stream_norm.hip", "ring_rows.hip", "window_prefill.hip",
           "window_prefill_latent.hip", "window_prefill_heads.hip", "window_decode.hip", "window_decode_split.hip", "post_norm.hip",
           "talk.hip", "talk_prefill.hip", "talk_decode.hip"]

HIPCC_FLAGS = [
    "--offload-arch=gfx950",
    "-O3",
    "-std=c++17",
    "-fPIC",
    "-fhip-fp32-correctly-rounded-divide-sqrt",   # INT8 scales/codes must match IEEE division
    "-fno-fast-math",
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    "-Wno-unused-command-line-argument",
]


def _hipcc() -> str:
    exe = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"
    if not os.path.exists(exe):
        raise RuntimeError("hipcc not found; cannot build libminivllm_amd.so")
    return exe


def _compile(src, verbose, extra=(), suffix=""):
    obj_dir = os.path.join(PKG_DIR, "build")
    os.makedirs(obj_dir, exist_ok=True)
    obj = os.path.join(obj_dir, src.replace(".hip", suffix + ".o"))
    cmd = [_hipcc(), *HIPCC_FLAGS, *extra, "-c", os.path.join(CSRC, src), "-o", obj]
    if verbose:
        print(" ".join(cmd), flush=True)
    res = subprocess.run(cmd, capture_output=True, text=True)
    err = "\n".join(l for l in res.stderr.splitlines() if "packed-fp32-ops" not in l)
    if res.returncode != 0:
        raise RuntimeError(f"hipcc failed for {src}:\n{err}")
    if verbose and err.strip():
        print(err, file=sys.stderr)
    return obj


def _link(lib, members, verbose):
    part = f"{lib}.{os.getpid()}"
    cmd = [_hipcc(), "--offload-arch=gfx950", "-shared", "-fPIC", "-o", part, *members]
    if verbose:
        print(" ".join(cmd), flush=True)
    res = subprocess.run(cmd, capture_output=True, text=True)
    if res.returncode != 0:
        raise RuntimeError(f"link failed:\n{res.stderr}")
    os.replace(part, lib)


def build_library(verbose: bool = True, jobs: int = 8) -> str:
    # the long ones first, so that no job is left compiling alone at the end
    order = sorted(SOURCES + PROBE_SOURCES, key=lambda src: -os.path.getsize(os.path.join(CSRC, src)))
    order.sort(key=lambda src: src not in ("prefill_other_dims.hip", "prefill_half_step_dims.hip", "paged_decode.hip"))
    with ThreadPoolExecutor(max_workers=jobs) as pool:
        running = {src: pool.submit(_compile, src, verbose) for src in order[:3]}
        # the probe library also holds the decode kernels built as "loads only" (the access pattern's ceiling)
        probe_decode = pool.submit(_compile, "paged_decode.hip", verbose, ("-DMVLLM_DECODE_LOADS_ONLY=1",), "_loads_only")
        # ... and the two-group prefill kernel with its per-tile clock stamps
        probe_prefill = pool.submit(_compile, "prefill_pingpong.hip", verbose, ("-DMVLLM_PP_TIMELINE=1",), "_timeline")
        running.update({src: pool.submit(_compile, src, verbose) for src in order[3:]})
        objs = {src: job.result() for src, job in running.items()}
        probes = [probe_decode.result(), probe_prefill.result()]
    _link(LIB_PATH, [objs[s] for s in SOURCES], verbose)
    _link(PROBE_LIB_PATH, [objs[s] for s in PROBE_SOURCES] + probes, verbose)
    return LIB_PATH


def part_path(sources) -> str:
    """Named after the sources' names and contents and the headers: a changed checkout builds another one."""
    digest = hashlib.sha1(" ".join(HIPCC_FLAGS).encode())
    headers = [f for f in os.listdir(CSRC) if f.endswith(".h")]
    for name in sorted([*sources, "absent_kernels.hip", *headers]):
        digest.update(name.encode())
        with open(os.path.join(CSRC, name), "rb") as f:
            digest.update(f.read())
    return os.path.join(PKG_DIR, f"libminivllm_part_{digest.hexdigest()[:10]}.so")


def build_part(sources, verbose: bool = False, jobs: int = 8) -> str:
    """A library of some of ``SOURCES``; kernel families it leaves out are replaced by stand-ins that take nothing."""
    with ThreadPoolExecutor(max_workers=jobs) as pool:
        objs = list(pool.map(lambda src: _compile(src, verbose, suffix="_part"), [*sources, "absent_kernels.hip"]))
    path = part_path(sources)
    _link(path, objs, verbose)
    return path


def ensure_library(sources, verbose: bool = False) -> str:
    """Path of a library that has ``sources``; the binding loads that one from now on."""
    from minivllm_amd import _C
    path = LIB_PATH
    if not os.path.exists(path):
        path = part_path(sources)
        if not os.path.exists(path):
            build_part(sources, verbose)
    _C.use_library(path)
    return path


if __name__ == "__main__":
    print(build_library())
