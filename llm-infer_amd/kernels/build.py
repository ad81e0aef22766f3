"""Compiles the HIP sources for gfx950 into shared libraries and loads them.

``libli_core.so`` holds every kernel of the softmax decoder whose sizes are run-time
values, ``libli_mixers.so`` those of the other mixers, norms and activations; the
attention kernels are compiled once per head size (``libli_attn_hd<N>.so``), at
the first call that needs that size.  Libraries are kept beside the sources (or in
a temporary folder when that is not writable) with a stamp of the sources they
were built from, and are rebuilt when the sources change.  There is no other
implementation behind these libraries: without them nothing runs.
"""
from __future__ import annotations

import ctypes
import hashlib
import os
import shutil
import subprocess
import sys
import tempfile
import threading
import time
from concurrent.futures import ThreadPoolExecutor

CSRC = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "csrc")
ARCH = "gfx950"
CORE_SOURCES = ("elementwise.hip", "gemm.hip", "gemm_prefill.hip", "sampling.hip")
ATTN_SOURCE = "attention.hip"
MIXER_SOURCES = ("mixers.hip",)
# the headers a library's sources include (its stamp covers them)
HEADERS = {"libli_core.so": ("common.h", "gemm_common.h", "no_alloc.h"), "libli_hybrid.so": ("common.h", "conv.h"),
           "libli_recurrent.so": ("common.h", "conv.h"), "libli_experts.so": ("common.h", "gemm_common.h")}
DEFAULT_HEADERS = ("common.h",)
FLAGS = ["--offload-arch=" + ARCH, "-O3", "-std=c++17", "-fPIC",
         "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops", "-Wno-unused-command-line-argument"]

_lock = threading.Lock()
_loaded: dict = {}


class BuildError(RuntimeError):
    pass


def _say(msg: str) -> None:
    print(f"[llm_infer_amd] {msg}", file=sys.stderr, flush=True)


def _preferred_dir() -> str:
    return os.environ.get("LLM_INFER_AMD_BUILD_DIR") or os.path.join(CSRC, "_build")


def build_dir() -> str:
    """Where libraries are built: the preferred folder, or one under the temporary folder if that
    cannot be written (a checkout that belongs to someone else)."""
    d = _preferred_dir()
    try:
        os.makedirs(d, exist_ok=True)
        fd, probe = tempfile.mkstemp(prefix=".w", dir=d)       # a name of its own: builds run side by side
        os.close(fd)
        os.remove(probe)
        return d
    except OSError:
        d = os.path.join(tempfile.gettempdir(), f"llm_infer_amd_build_{os.getuid()}")
        os.makedirs(d, exist_ok=True)
        return d


def _hipcc() -> str:
    for cand in (os.environ.get("HIPCC"), shutil.which("hipcc"), "/opt/rocm/bin/hipcc"):
        if cand and os.path.isfile(cand):
            return cand
    raise BuildError("hipcc not found: the HIP kernels cannot be built and there is no other implementation")


def _stamp(sources, defines, lib_name="") -> str:
    h = hashlib.sha256()
    for name in tuple(sources) + HEADERS.get(lib_name, DEFAULT_HEADERS):
        with open(os.path.join(CSRC, name), "rb") as f:
            h.update(name.encode() + b"\0" + f.read())
    h.update(" ".join(FLAGS + list(defines)).encode())
    return h.hexdigest()


def _run(cmd, what):
    env = dict(os.environ)
    env.setdefault("HOME", tempfile.gettempdir())            # hipcc wants a home for its temporary files
    t0 = time.time()
    proc = subprocess.Popen(cmd, stdout=subprocess.PIPE, stderr=subprocess.STDOUT, text=True, env=env)
    done = threading.Event()

    def ticker():
        while not done.wait(20.0):
            _say(f"still compiling {what} ({time.time() - t0:.0f} s)")
    th = threading.Thread(target=ticker, daemon=True)
    th.start()
    out, _ = proc.communicate()
    done.set()
    if proc.returncode != 0:
        raise BuildError(f"compiling {what} failed:\n{' '.join(cmd)}\n{out}")
    return out


# Kernels that count their own loads in flight (waits placed by hand): a register spilled by the compiler
# would be a load that they do not count, so a build in which they use scratch memory is refused.
# (gemm_wreg: W into a ring of registers by global_load_dwordx4; attn_prefill: the fragments of a page out of
# LDS by ds_read_b128; both written as instructions whose results the compiler knows nothing about until the
# hand-counted wait.)
NO_SCRATCH = {"gemm_prefill.hip": "gemm_wreg_kernel", "attention.hip": "attn_prefill_kernel"}


def _check_no_scratch(report: str, kernel: str, src: str) -> None:
    """``report``: the compiler's resource remarks (-Rpass-analysis=kernel-resource-usage)."""
    name, seen = None, 0
    for line in report.splitlines():
        if "Function Name:" in line:
            name = line.split("Function Name:")[1].split()[0]
        elif "ScratchSize [bytes/lane]:" in line and name and kernel in name:
            seen += 1
            size = int(line.split("ScratchSize [bytes/lane]:")[1].split()[0])
            if size != 0:
                raise BuildError(f"{src}: {name} uses {size} bytes of scratch memory a lane; its waits count on none")
    if seen == 0:
        raise BuildError(f"{src}: the compiler reported no resource usage for {kernel}")


def _build_library(lib_name: str, sources, defines=(), force=False) -> str:
    stamp = _stamp(sources, defines, lib_name)
    if not force:
        # a library built from these very sources is taken where it lies, also from a folder that
        # cannot be written
        for d in dict.fromkeys((_preferred_dir(), build_dir())):
            lib = os.path.join(d, lib_name)
            if os.path.isfile(lib) and os.path.isfile(lib + ".stamp"):
                with open(lib + ".stamp") as f:
                    if f.read().strip() == stamp:
                        return lib
    d = build_dir()
    lib = os.path.join(d, lib_name)
    stamp_file = lib + ".stamp"
    hipcc = _hipcc()
    _say(f"compiling {lib_name} for {ARCH} ...")
    t0 = time.time()
    tag = f"{os.getpid()}_{threading.get_ident()}"
    objs = []

    def compile_one(src):
        obj = os.path.join(d, f"{lib_name}.{src}.{tag}.o")
        report = ["-Rpass-analysis=kernel-resource-usage"] if src in NO_SCRATCH else []
        out = _run([hipcc, *FLAGS, *defines, *report, "-c", os.path.join(CSRC, src), "-o", obj], f"{lib_name}:{src}")
        if report:
            _check_no_scratch(out, NO_SCRATCH[src], src)
        return obj
    try:
        with ThreadPoolExecutor(max_workers=min(4, len(sources))) as pool:
            objs = list(pool.map(compile_one, sources))
        tmp = lib + f".{tag}.tmp"
        _run([hipcc, "--offload-arch=" + ARCH, "-shared", "-fPIC", "-o", tmp, *objs], f"{lib_name} (link)")
        os.replace(tmp, lib)
        with open(stamp_file, "w") as f:
            f.write(stamp)
    finally:
        for o in objs:
            if os.path.isfile(o):
                os.remove(o)
    _say(f"built {lib_name} in {time.time() - t0:.0f} s")
    return lib


def _load(lib_name, sources, defines=(), force=False):
    with _lock:
        if not force and lib_name in _loaded:
            return _loaded[lib_name]
        import torch  # noqa: F401  (the HIP runtime must be the one torch has loaded)
        path = _build_library(lib_name, sources, defines, force)
        _loaded[lib_name] = ctypes.CDLL(path)
        return _loaded[lib_name]


def core_library(force=False):
    return _load("libli_core.so", CORE_SOURCES, (), force)


def attention_library(head_dim: int, force=False):
    if head_dim % 16 != 0 or not 16 <= head_dim <= 256:
        raise BuildError(f"head size {head_dim}: the attention kernels take multiples of 16 up to 256")
    return _load(f"libli_attn_hd{head_dim}.so", (ATTN_SOURCE,), (f"-DHEAD_DIM={head_dim}",), force)


def mixers_library(force=False):
    """The kernels of the other mixers and arrangements (csrc/mixers.hip): a library of its own, so that a
    model is not kept waiting for kernels that it does not run."""
    return _load("libli_mixers.so", MIXER_SOURCES, (), force)


HYBRID_SOURCES = ("hybrid.hip", "latent.hip", "gated.hip")


def hybrid_library(force=False):
    """The kernels of hybrid decoders (csrc/hybrid.hip: differential attention over blocks of positions, the
    state-space recurrence and its convolution, the experts' router; csrc/latent.hip: latent attention's
    preparation and products per head, the matrix-memory recurrence, the bigram embedding, the depth-weighted
    average of the residual stream; csrc/gated.hip: the norm of a sub-layer's output with the residual sum, the rotation
    of half-paired dimensions with the cache write, the clamped gated activation, experts by table): a library of its own,
    as the mixers' is."""
    return _load("libli_hybrid.so", HYBRID_SOURCES, (), force)


RECURRENT_SOURCES = ("recurrent.hip", "recurrent_chunks.hip")


def recurrent_library(force=False):
    """The recurrent mixers' kernels (csrc/recurrent.hip, and csrc/recurrent_chunks.hip for prompts: the gated delta rule, the selective scan with a decay for every
    channel and state, time mixing with a decay for every key channel): a library of its own, as the mixers' is."""
    return _load("libli_recurrent.so", RECURRENT_SOURCES, (), force)


EXPERT_SOURCES = ("experts.hip",)


def experts_library(force=False):
    """Routed experts by pairs of token and expert (csrc/experts.hip: the router, the sorted pairs, the products of few
    pairs, their sum): a library of its own, as the mixers' is."""
    return _load("libli_experts.so", EXPERT_SOURCES, (), force)


DIFF_ATTN_SOURCE = "diff_attention.hip"


def _diff_attention_args(map_dim: int, value_dim: int):
    if map_dim % 16 != 0 or not 16 <= map_dim <= 256 or value_dim % 32 != 0 or not 32 <= value_dim <= 256:
        raise BuildError(f"head sizes {map_dim} / {value_dim}: the differential attention kernel takes a map size that is "
                         "a multiple of 16 and a value size that is a multiple of 32, both up to 256")
    return (f"libli_diffattn_k{map_dim}_v{value_dim}.so", (DIFF_ATTN_SOURCE,),
            (f"-DMAP_DIM={map_dim}", f"-DVALUE_DIM={value_dim}"))


def diff_attention_library(map_dim: int, value_dim: int, force=False):
    """The matrix-core kernel of differential attention for one pair of sizes (a map's keys, values), compiled at
    the first call that needs the pair."""
    return _load(*_diff_attention_args(map_dim, value_dim), force)


SIGMOID_ATTN_SOURCE = "sigmoid_attention.hip"


def _sigmoid_attention_args(key_dim: int, value_dim: int):
    for n in (key_dim, value_dim):
        if n % 16 != 0 or not 16 <= n <= 256:
            raise BuildError(f"head size {n}: the sigmoid attention kernels take multiples of 16 up to 256")
    return (f"libli_sigattn_k{key_dim}_v{value_dim}.so", (SIGMOID_ATTN_SOURCE,),
            (f"-DKEY_DIM={key_dim}", f"-DVALUE_DIM={value_dim}"))


def sigmoid_attention_library(key_dim: int, value_dim: int, force=False):
    """The matrix-core kernels of sigmoid attention for one pair of head sizes (keys, values), compiled at the
    first call that needs the pair."""
    return _load(*_sigmoid_attention_args(key_dim, value_dim), force)


def build_all(head_dims=(16, 32, 48, 64, 128), force=True, sigmoid_head_dims=((48, 32), (128, 128)),
              diff_head_dims=((32, 64), (64, 128))) -> None:
    """Compile the core library, the mixers' library, the attention library for each head size given and the
    sigmoid attention library for each pair of head sizes given."""
    core_library(force=force)
    mixers_library(force=force)
    hybrid_library(force=force)
    recurrent_library(force=force)
    experts_library(force=force)
    with ThreadPoolExecutor(max_workers=4) as pool:
        list(pool.map(lambda p: _build_library(*_sigmoid_attention_args(*p), force), sigmoid_head_dims))
        list(pool.map(lambda p: _build_library(*_diff_attention_args(*p), force), diff_head_dims))
    with ThreadPoolExecutor(max_workers=4) as pool:
        list(pool.map(lambda hd: _build_library(f"libli_attn_hd{hd}.so", (ATTN_SOURCE,),
                                                (f"-DHEAD_DIM={hd}",), force), head_dims))
