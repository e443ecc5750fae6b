"""Build the HIP libraries in-tree with hipcc for gfx950 (cross-compiles without a GPU).

  libomni_talker.so        the product: HIP kernels + the C-ABI of include/omni_talker.h, policy knobs compiled in
  libomni_decoder.so       the kernels of the decoder-only language models (include/omni_decoder.h): its own few sources plus the large-M GEMM and
                           the sampler both libraries link
  libomni_talker_debug.so  the talker's sources with -DOMNI_DEBUG_HOOKS (run-time policy knobs, omni_debug_* setters) plus
                           csrc/debug.hip (launch / memory-system probes): scripts/ and the tile-sweep tests only

All are git-ignored but travel with the repo snapshot.  `sources_digest()` is stamped into a side file next to each
library so that _lib.load() can refuse a library that is older than csrc/.
"""
from __future__ import annotations

import hashlib
import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
LIB = os.path.join(HERE, "libomni_talker.so")
LIB_DECODER = os.path.join(HERE, "libomni_decoder.so")
LIB_DEBUG = os.path.join(HERE, "libomni_talker_debug.so")
SOURCES = ["errors.hip", "capi.hip", "gemm.hip", "gemm_prefill.hip", "norm.hip", "rope_kv.hip", "paged_attn.hip", "prefill_attn.hip", "moe.hip",
           "sampler.hip", "cp_chain.hip", "bb_chain.hip", "moe_chain.hip", "allreduce.hip", "codec.hip", "conv_unit.hip"]
DECODER_SOURCES = ["errors.hip", "gemm_prefill.hip", "sampler.hip", "decoder_rows.hip", "gemm_stream.hip", "head_gemm.hip", "latent_attn.hip",
                   "window_attn.hip", "decay_rec.hip"]
# debug library only: the probes, and the losing A/B arms of the backbone chain (no product knob reaches them)
DEBUG_ONLY = ["debug.hip", "bb_engine.hip", "bb_all.hip"]
# per-file extra flags
EXTRA = {"debug.hip": ["-mllvm", "-amdgpu-kernarg-preload-count=16"]}
HIPCC = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
FLAGS = ["--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-Wall", "-Wno-unused-function",
         "-fno-gpu-rdc",
         # no packed fp32 (v_pk_fma / mul / add_f32): hipcc forms them from ordinary float code, and some of their operand forms have returned
         # wrong values beside another wave's MFMAs (tests/test_build_rules.py)
         "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def _headers() -> list[str]:
    hdrs = [os.path.join(CSRC, f) for f in sorted(os.listdir(CSRC)) if f.endswith((".cuh", ".h"))]
    inc = os.path.normpath(os.path.join(HERE, "..", "include"))      # every ABI header: a struct change in any of them is a new library
    hdrs += [os.path.join(inc, f) for f in sorted(os.listdir(inc)) if f.endswith(".h")]
    return hdrs


def sources_digest(debug: bool = False, sources: list[str] | None = None) -> str:
    """sha256 over every file the library is built from (+ the flags): what _lib.load() compares the stamp with."""
    h = hashlib.sha256()
    names = [s for s in (sources or SOURCES + (DEBUG_ONLY if debug else [])) if os.path.exists(os.path.join(CSRC, s))]
    for f in [os.path.join(CSRC, s) for s in names] + _headers():
        h.update(os.path.basename(f).encode())
        h.update(open(f, "rb").read())
    h.update(" ".join(FLAGS).encode())
    h.update(repr(sorted(EXTRA.items())).encode())
    return h.hexdigest()


def _stale(out: str, deps: list[str]) -> bool:
    if not os.path.exists(out):
        return True
    t = os.path.getmtime(out)
    return any(os.path.getmtime(d) > t for d in deps)


def _run(cmd, verbose=False):
    r = subprocess.run(cmd, capture_output=True, text=True)
    if r.returncode != 0:
        raise RuntimeError("hipcc failed: %s\n%s" % (" ".join(cmd), r.stderr))
    if verbose and r.stderr:
        print(r.stderr, file=sys.stderr)


def _build_one(lib: str, sources: list[str], objdir: str, extra: list[str], force: bool, verbose: bool, digest: str) -> str:
    hdrs = _headers()
    os.makedirs(objdir, exist_ok=True)
    sources = [s for s in sources if os.path.exists(os.path.join(CSRC, s))]
    # objects of other flags are stale whatever their age
    flag_file, flags = os.path.join(objdir, "flags"), repr((HIPCC, FLAGS, extra, sorted(EXTRA.items())))
    if not os.path.exists(flag_file) or open(flag_file).read() != flags:
        force = True
    jobs = []
    for s in sources:
        src = os.path.join(CSRC, s)
        obj = os.path.join(objdir, s.replace(".hip", ".o"))
        if force or _stale(obj, [src] + hdrs):
            jobs.append([HIPCC, *FLAGS, *extra, *EXTRA.get(s, []), "-c", src, "-o", obj])
    with ThreadPoolExecutor(max_workers=4) as ex:
        list(ex.map(lambda c: _run(c, verbose), jobs))
    with open(flag_file, "w") as f:
        f.write(flags)
    objs = [os.path.join(objdir, s.replace(".hip", ".o")) for s in sources]
    stamp = lib + ".digest"
    old = open(stamp).read().strip() if os.path.exists(stamp) else ""
    if force or jobs or _stale(lib, objs) or old != digest:
        _run([HIPCC, "--offload-arch=gfx950", "-shared", "-fPIC", "-o", lib, *objs], verbose)
        with open(stamp, "w") as f:
            f.write(digest + "\n")
    return lib


def build(force: bool = False, verbose: bool = False, debug: bool = True) -> str:
    lib = _build_one(LIB, SOURCES, os.path.join(HERE, "build"), [], force, verbose, sources_digest(False))
    build_decoder(force, verbose, shared_fresh=True)
    if debug:
        _build_one(LIB_DEBUG, SOURCES + DEBUG_ONLY, os.path.join(HERE, "build", "debug"), ["-DOMNI_DEBUG_HOOKS"], force, verbose,
                   sources_digest(True))
    return lib


def build_decoder(force: bool = False, verbose: bool = False, shared_fresh: bool = False) -> str:
    """The language-model library alone (what a process that serves no talker needs).  shared_fresh: the objects it shares with the talker's
    library were just compiled."""
    if force and shared_fresh:
        for s in DECODER_SOURCES:
            obj = os.path.join(HERE, "build", s.replace(".hip", ".o"))
            if s not in SOURCES and os.path.exists(obj):
                os.remove(obj)
        force = False
    return _build_one(LIB_DECODER, DECODER_SOURCES, os.path.join(HERE, "build"), [], force, verbose, sources_digest(sources=DECODER_SOURCES))


def ensure_decoder() -> str:
    """libomni_decoder.so of the sources that are here: compiled when absent or older (one process at a time)."""
    import fcntl
    os.makedirs(os.path.join(HERE, "build"), exist_ok=True)
    with open(os.path.join(HERE, "build", "decoder.lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        stamp = LIB_DECODER + ".digest"
        if not (os.path.exists(LIB_DECODER) and os.path.exists(stamp) and open(stamp).read().strip() == sources_digest(sources=DECODER_SOURCES)):
            build_decoder()
    return LIB_DECODER


if __name__ == "__main__":
    print(build(force="--force" in sys.argv, verbose=True))
