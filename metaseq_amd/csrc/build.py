"""Builds the shared libraries for gfx950 with hipcc (no GPU needed: hipcc cross-compiles).

    core    libmetaseq_amd.so     OPT decoder, selection and sampling (include/metaseq_amd.h)
    hybrid  libmetaseq_hybrid.so  hybrid decoders: latent and grouped attention, recurrent layers,
                                  routed feed-forwards (include/metaseq_hybrid.h)

Usage: python -m metaseq_amd.csrc.build [core|hybrid ...]
"""
import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
LIBS = {"core": os.path.join(HERE, "libmetaseq_amd.so"),
        "hybrid": os.path.join(HERE, "libmetaseq_hybrid.so")}
LIB = LIBS["core"]
SOURCES = {
    "core": ["capi.hip", "layernorm.hip", "embed.hip", "gemm.hip", "attention.hip",
             "attention_prefill.hip", "sampling.hip", "probe.hip", "decoder_step.hip"],
    "hybrid": ["capi.hip", "gemm_bf16.hip", "gemm_bf16_post.hip", "group_linear.hip", "moe.hip",
               "rmsnorm.hip", "recurrent.hip", "latent_attention.hip", "grouped_attention.hip",
               "hybrid_step.hip"],
}
HEADERS = ["common.h", "gemm_kernels.h", "attention_tiles.h",
           os.path.join("..", "..", "include", "metaseq_amd.h"),
           os.path.join("..", "..", "include", "metaseq_hybrid.h")]
FLAGS = [
    "--offload-arch=gfx950", "-O3", "-fPIC", "-std=c++17", "-Wall", "-Wno-unused-function",
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
]


# per-source extras.  The flash-style attention kernels keep their MFMA results in ordinary vector
# registers (their softmax reads every score; by default hipcc parks them in the accumulator bank
# and copies each one out)
EXTRA_FLAGS = {"attention_prefill.hip": ["-mllvm", "-amdgpu-mfma-vgpr-form=1"],
               "latent_attention.hip": ["-mllvm", "-amdgpu-mfma-vgpr-form=1"],
               "grouped_attention.hip": ["-mllvm", "-amdgpu-mfma-vgpr-form=1"]}


def _hipcc():
    for c in (os.environ.get("HIPCC"), "/opt/rocm/bin/hipcc", "hipcc"):
        if c and (os.path.sep not in c or os.path.exists(c)):
            return c
    raise RuntimeError("hipcc not found")


def needs_build(component="core"):
    lib = LIBS[component]
    if not os.path.exists(lib):
        return True
    t = os.path.getmtime(lib)
    return any(os.path.getmtime(os.path.join(HERE, d)) > t for d in SOURCES[component] + HEADERS)


def build(force=True, verbose=True, components=("core", "hybrid")):
    """Compiles the sources of the named components and links their shared libraries in-tree.
    Without ``force`` a component whose library is newer than its sources is left alone."""
    components = [c for c in components if force or needs_build(c)]
    if not components:
        return LIB
    hipcc = _hipcc()
    objdir = os.path.join(HERE, "build")
    os.makedirs(objdir, exist_ok=True)

    def compile_one(src):
        obj = os.path.join(objdir, src.replace(".hip", ".o"))
        cmd = [hipcc] + FLAGS + EXTRA_FLAGS.get(src, []) + ["-c", os.path.join(HERE, src), "-o", obj]
        r = subprocess.run(cmd, capture_output=True, text=True)
        err = "\n".join(l for l in r.stderr.splitlines()
                        if "packed-fp32-ops" not in l)  # host pass does not know the feature
        if r.returncode != 0:
            raise RuntimeError("hipcc failed for %s:\n%s" % (src, err))
        if verbose and err.strip():
            print(err, file=sys.stderr)
        return obj

    sources = sorted({src for c in components for src in SOURCES[c]})
    with ThreadPoolExecutor(max_workers=min(8, len(sources))) as ex:
        objs = dict(zip(sources, ex.map(compile_one, sources)))
    for c in components:
        # linked under another name and moved into place: a reader never sees half a library
        part = LIBS[c] + ".part"
        cmd = ([hipcc, "--offload-arch=gfx950", "-shared", "-fPIC", "-Wl,-Bsymbolic", "-o", part]
               + [objs[src] for src in SOURCES[c]])
        r = subprocess.run(cmd, capture_output=True, text=True)
        if r.returncode != 0:
            raise RuntimeError("link failed:\n" + r.stderr)
        os.replace(part, LIBS[c])
        if verbose:
            print("built", LIBS[c])
    return LIB


if __name__ == "__main__":
    build(force=True, components=sys.argv[1:] or ("core", "hybrid"))
