"""Build the C-ABI libraries of HIP kernels in-tree for gfx950: libtrimkv_hip.so (the TRIM-KV cache path and its decoders),
libtrimkv_hybrid.so (what the hybrid decoders share, windowed attention), libtrimkv_mlstm.so and libtrimkv_moe.so (their
recurrent layers and routed experts).

Usage: ``python -m trimkv_amd.build [--changed] [hip|hybrid|mlstm|moe ...]`` (hipcc cross-compiles without a GPU; ``--changed``
recompiles only the sources whose object file is older than its inputs; no name: all of them).
"""
from __future__ import annotations

import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
INCLUDE = os.path.join(os.path.dirname(HERE), "include")
LIB_PATH = os.path.join(HERE, "libtrimkv_hip.so")
SOURCES = ["api.hip", "append.hip", "evict.hip", "attn_decode.hip", "attn_decode_append.hip", "attn_decode_pieces.hip", "attn_decode_append_pieces.hip", "attn_decode_append_gated.hip", "attn_decode_append_pieces_gated.hip", "pieces_plan.hip", "attn_prefill.hip", "gate.hip", "stream_probe.hip", "decoder_ops.hip"]
HYBRID_SOURCES = ["hybrid_ops.hip", "window_attn.hip", "window_decode.hip"]
LIBRARIES = {"hip": (LIB_PATH, SOURCES), "hybrid": (os.path.join(HERE, "libtrimkv_hybrid.so"), HYBRID_SOURCES),
             "mlstm": (os.path.join(HERE, "libtrimkv_mlstm.so"), ["mlstm.hip"]), "moe": (os.path.join(HERE, "libtrimkv_moe.so"), ["moe.hip"])}

HIPCC_FLAGS = [
    "--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-I" + INCLUDE, "-I" + CSRC,
    # packed fp32 VALU ops are kept out of every kernel in this library
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    "-Wno-unused-value",
]
# maxima of scores: without this every operand of fmaxf is first run through v_max_f32 to quiet a NaN that cannot be there
# (the decode kernel is scheduled worse with it: 246 against 185 us at 64 x 8 heads of 4096 rows)
EXTRA_FLAGS = {"window_attn.hip": ["-fno-honor-nans"]}


def _run(cmd):
    proc = subprocess.run(cmd, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True)
    out = "\n".join(l for l in proc.stdout.splitlines() if "packed-fp32-ops" not in l)
    if proc.returncode != 0:
        raise RuntimeError("command failed: %s\n%s" % (" ".join(cmd), out))
    return out


def _stale(src: str, obj: str) -> bool:
    """An object is stale when its source, any header beside it or the public header is newer."""
    if not os.path.exists(obj):
        return True
    deps = [os.path.join(CSRC, src)] + [os.path.join(CSRC, f) for f in os.listdir(CSRC) if f.endswith(".h")]
    deps += [os.path.join(INCLUDE, f) for f in os.listdir(INCLUDE)]
    return any(os.path.getmtime(d) > os.path.getmtime(obj) for d in deps)


def build(verbose: bool = True, only_changed: bool = False, libraries=tuple(LIBRARIES)) -> str:
    """Compile every source of the named libraries (or, with ``only_changed``, the ones whose object is older than its
    inputs) and link them."""
    hipcc = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
    objdir = os.path.join(HERE, "build")
    os.makedirs(objdir, exist_ok=True)
    obj_of = lambda s: os.path.join(objdir, s.replace(".hip", ".o"))
    srcs = [s for name in libraries for s in LIBRARIES[name][1]]
    if only_changed:
        srcs = [s for s in srcs if _stale(s, obj_of(s))]

    def compile_one(src):
        return _run([hipcc] + HIPCC_FLAGS + EXTRA_FLAGS.get(src, []) + ["-c", os.path.join(CSRC, src), "-o", obj_of(src)])

    if srcs:
        with ThreadPoolExecutor(max_workers=min(os.cpu_count() or 4, 8, len(srcs))) as ex:
            for src, out in zip(srcs, ex.map(compile_one, srcs)):
                if verbose and out.strip():
                    print("[%s]\n%s" % (src, out))
    for name in libraries:
        path, sources = LIBRARIES[name]
        part = "%s.%d" % (path, os.getpid())       # linked beside and renamed: nobody loads half a library
        _run([hipcc, "--offload-arch=gfx950", "-shared", "-fPIC", "-o", part] + [obj_of(s) for s in sources])
        os.replace(part, path)
        if verbose:
            print("built", path)
    return LIBRARIES[libraries[-1]][0]


def ensure(libraries) -> None:
    """Build those of the named libraries that are not there (a fresh checkout)."""
    missing = tuple(n for n in libraries if not os.path.exists(LIBRARIES[n][0]))
    if missing:
        build(verbose=False, only_changed=True, libraries=missing)


if __name__ == "__main__":
    names = [a for a in sys.argv[1:] if not a.startswith("--")]
    build(only_changed="--changed" in sys.argv[1:], libraries=tuple(names) or tuple(LIBRARIES))
    sys.exit(0)
