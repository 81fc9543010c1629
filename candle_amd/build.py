"""Builds libcandle_hip_quant.so (gfx950) in-tree with hipcc.

    python -m candle_amd.build            # compile what changed, link
    python -m candle_amd.build --force    # recompile everything
    python -m candle_amd.build --mixer    # only libcandle_hip_mixer.so (what models with bfloat16 weights run on)

hipcc cross-compiles for gfx950 without a GPU present.  Flags:
  -ffp-contract=off   the quantizers and the dequantizer must round exactly like the scalar CPU code
                      (kernels that want an FMA call fmaf explicitly);
  -packed-fp32-ops    disabled: hipcc must not form packed-f32 instructions from scalar float code;
  -amdgpu-kernarg-preload-count=14   the first fourteen dwords of scalar kernel arguments are placed in SGPRs at wave
                      launch (kernels keep an entry that loads them for firmware without the feature).
"""
from __future__ import annotations

import concurrent.futures
import os
import subprocess
import sys

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
OBJ = os.path.join(CSRC, "obj")
LIB = os.path.join(HERE, "libcandle_hip_quant.so")

LIB_MIXER = os.path.join(HERE, "libcandle_hip_mixer.so")
LIB_BENCH = os.path.join(HERE, "libcq_bench.so")

SOURCES = ["cq_api.hip", "cq_dequant.hip", "cq_actquant.hip", "cq_matvec.hip", "cq_matmul.hip", "cq_moe.hip", "cq_quantize.hip", "cq_nn.hip", "cq_layer.hip", "cq_matvec_batch.hip", "cq_status.hip"]
# models with bfloat16 weights: dense products and sequence mixers, with the glue of cq_nn.hip; complete without the library above, so
# that such a model can run without compiling the quantized kernels
MIXER_SOURCES = ["cq_nn.hip", "cq_status.hip", "cq_dense.hip", "cq_mix_glue.hip", "cq_mix_attention.hip", "cq_mix_state.hip", "cq_mix_latent.hip", "cq_mix_moe.hip"]
MIXER_HEADERS = ("candle_hip_mixer.h", "cq_mix.h", "cq_dense.h")
# the benchmark's plain-read yardstick kernel: a library of its own, not part of the C ABI
BENCH_SOURCES = ["cq_bench.hip"]

HIPCC = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
FLAGS = [
    "--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-ffp-contract=off",
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    "-mllvm", "-amdgpu-kernarg-preload-count=14",
    "-Wall", "-Wno-unused-function", "-Wno-unknown-warning-option",
]


def _headers_mtime(src: str) -> float:
    hs = [os.path.join(CSRC, f) for f in os.listdir(CSRC) if f.endswith(".h")]
    inc = os.path.join(os.path.dirname(HERE), "include")
    hs += [os.path.join(inc, f) for f in os.listdir(inc) if f.endswith(".h")]
    if src.startswith(("cq_mix", "cq_dense")):
        return max(os.path.getmtime(h) for h in hs)
    return max(os.path.getmtime(h) for h in hs if os.path.basename(h) not in MIXER_HEADERS)


def _compile(src: str, force: bool) -> str:
    obj = os.path.join(OBJ, src.replace(".hip", ".o"))
    path = os.path.join(CSRC, src)
    if not force and os.path.exists(obj) and os.path.getmtime(obj) > max(os.path.getmtime(path), _headers_mtime(src)):
        return obj
    tmp = f"{obj}.{os.getpid()}.o"
    cmd = [HIPCC, *FLAGS, "-c", path, "-o", tmp]
    r = subprocess.run(cmd, capture_output=True, text=True)
    err = "\n".join(l for l in r.stderr.splitlines() if "packed-fp32-ops" not in l)
    if r.returncode != 0:
        raise RuntimeError(f"hipcc failed for {src}:\n{err}")
    if err.strip():
        sys.stderr.write(err + "\n")
    os.replace(tmp, obj)
    return obj


def _build(groups, force: bool) -> None:
    """Compile the sources of all (library, sources) pairs side by side, then link the libraries that are out of date."""
    os.makedirs(OBJ, exist_ok=True)
    if not force:                  # a library newer than everything it is made of needs no objects
        newest = lambda s: max(os.path.getmtime(os.path.join(CSRC, s)), _headers_mtime(s))
        groups = [(lib, ss) for lib, ss in groups if not os.path.exists(lib) or os.path.getmtime(lib) <= max(newest(s) for s in ss)]
        if not groups:
            return
    srcs = list(dict.fromkeys(s for _, sources in groups for s in sources))
    with concurrent.futures.ThreadPoolExecutor(max_workers=min(8, len(srcs))) as ex:
        objs = dict(zip(srcs, ex.map(lambda s: _compile(s, force), srcs)))
    for lib, sources in groups:
        lobjs = [objs[s] for s in sources]
        if force or not os.path.exists(lib) or any(os.path.getmtime(o) > os.path.getmtime(lib) for o in lobjs):
            tmp = f"{lib}.{os.getpid()}"
            r = subprocess.run([HIPCC, "--offload-arch=gfx950", "-shared", "-fPIC", "-o", tmp, *lobjs], capture_output=True, text=True)
            if r.returncode != 0:
                raise RuntimeError("link failed:\n" + r.stderr)
            os.replace(tmp, lib)


def build(force: bool = False) -> str:
    _build(((LIB, SOURCES), (LIB_MIXER, MIXER_SOURCES), (LIB_BENCH, BENCH_SOURCES)), force)
    return LIB


def build_mixer(force: bool = False) -> str:
    _build(((LIB_MIXER, MIXER_SOURCES),), force)
    return LIB_MIXER


if __name__ == "__main__":
    print((build_mixer if "--mixer" in sys.argv else build)(force="--force" in sys.argv))
