"""Builds the package's libraries for gfx950 with hipcc (no torch headers, no cmake).

    python -m nanochat_amd.build [gpt | stack]

Two libraries, so that a process builds and loads what its model needs: `gpt` (libnanochat_amd.so: the FP8 GPT, sampling, quantization)
and `stack` (libnanochat_amd_stack.so: decoders made of configured layers).  They are written next to this file so they travel with the
source tree.
"""
import fcntl
import hashlib
import os
import subprocess
import sys
from concurrent.futures import ThreadPoolExecutor

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
INCLUDE = os.path.join(os.path.dirname(HERE), "include")
OBJ_DIR = os.path.join(HERE, "_build")

SOURCES = ["nc_api.hip", "nc_host.hip", "nc_quantize.hip", "nc_gemm.hip", "nc_elementwise.hip", "nc_attention.hip", "nc_attention_prefill.hip",
           "nc_sample.hip", "nc_forward.hip", "nc_profile.hip", "nc_gemm_decode.hip"]
STACK_SOURCES = ["nc_stack_forward.hip", "nc_host.hip", "nc_stack_gemm.hip", "nc_stack_rows.hip", "nc_latent_attention.hip", "nc_retention.hip",
                 "nc_window_attention.hip", "nc_selective_scan.hip", "nc_profile.hip"]
TARGETS = {"gpt": ("libnanochat_amd.so", SOURCES), "stack": ("libnanochat_amd_stack.so", STACK_SOURCES)}
LIB_PATH = os.path.join(HERE, TARGETS["gpt"][0])


def lib_path(target="gpt"):
    return os.path.join(HERE, TARGETS[target][0])


def stamp_path(target="gpt"):
    """Digest of what the library was built from."""
    return lib_path(target) + ".sources"


STAMP_PATH = stamp_path()

# -packed-fp32-ops off: packed fp32 VALU forms are not to be generated on this hardware pool
FLAGS = ["--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-Wall", "-Wno-unused-function",
         "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]


def sources_digest(target="gpt"):
    """SHA-256 over the flags and every file the library is compiled from."""
    h = hashlib.sha256(" ".join(FLAGS).encode())
    files = [os.path.join(CSRC, f) for f in sorted(TARGETS[target][1])]
    files += [os.path.join(CSRC, f) for f in sorted(os.listdir(CSRC)) if f.endswith(".h")]
    files += [os.path.join(INCLUDE, f) for f in sorted(os.listdir(INCLUDE)) if f.endswith(".h")]
    for f in files:
        h.update(os.path.basename(f).encode())
        h.update(open(f, "rb").read())
    return h.hexdigest()


def is_current(target):
    """Whether the library is there and was built from these sources."""
    path = stamp_path(target)
    return os.path.exists(lib_path(target)) and os.path.exists(path) and open(path).read().strip() == sources_digest(target)


def _compile(src):
    obj = os.path.join(OBJ_DIR, src.replace(".hip", ".o"))
    cmd = ["hipcc", *FLAGS, "-c", os.path.join(CSRC, src), "-o", obj]
    r = subprocess.run(cmd, capture_output=True, text=True)
    return src, obj, r


def _build(targets, verbose):
    for t in targets:
        if os.path.exists(stamp_path(t)):
            os.remove(stamp_path(t))              # a failed build must not leave a stamp that matches
    sources = sorted({src for t in targets for src in TARGETS[t][1]})
    with ThreadPoolExecutor(max_workers=min(8, len(sources))) as ex:
        results = list(ex.map(_compile, sources))
    objs = {}
    for src, obj, r in results:
        noise = [l for l in r.stderr.splitlines() if "packed-fp32-ops" not in l and l.strip()]
        if r.returncode != 0:
            raise RuntimeError(f"hipcc failed on {src}:\n{r.stderr}")
        if verbose and noise:
            print(f"[{src}]\n" + "\n".join(noise), file=sys.stderr)
        objs[src] = obj
    for t in targets:
        part = f"{lib_path(t)}.{os.getpid()}.tmp"
        link = ["hipcc", "--offload-arch=gfx950", "-shared", "-fPIC", "-Wl,--no-undefined", "-o", part, *(objs[src] for src in TARGETS[t][1])]
        r = subprocess.run(link, capture_output=True, text=True)
        if r.returncode != 0:
            raise RuntimeError(f"link failed:\n{r.stderr}")
        os.replace(part, lib_path(t))             # (a process that has the old library mapped keeps it)
        with open(stamp_path(t), "w") as f:
            f.write(sources_digest(t) + "\n")


def _locked():
    os.makedirs(OBJ_DIR, exist_ok=True)
    lock = open(os.path.join(OBJ_DIR, "lock"), "w")
    fcntl.flock(lock, fcntl.LOCK_EX)              # one build at a time in this tree; released when the file is closed
    return lock


def build(verbose=True, targets=tuple(TARGETS)):
    """Compile the given libraries, always; returns their paths."""
    with _locked():
        _build(targets, verbose)
    return [lib_path(t) for t in targets]


def ensure(target):
    """Compile one library unless it is there and current."""
    if not is_current(target):
        with _locked():
            if not is_current(target):            # somebody else may have built it meanwhile
                _build([target], verbose=False)
    return lib_path(target)


if __name__ == "__main__":
    print("\n".join(build(targets=tuple(sys.argv[1:]) or tuple(TARGETS))))
