"""Light native library for the hybrid-model kernels (grouped RMS norm, xIELU,
minGRU scan, general-size paged attention, shift norms, latent attention,
sum+norm residual step, q/k/v prep, head-mixed attention, matrix-state scan,
multi-stream residual step, grouped router and routed combine, layer norms,
fp32 projections onto a few columns, short convolutions, gated delta rule).

These kernels expose a plain C ABI and need no torch headers, so they are
compiled by direct ``hipcc`` calls (side by side, without the minutes the
torch extension takes) into ``llm_instance_gateway_amd/_hybrid.so`` and
loaded with ctypes.  A model that needs only these kernels can therefore be
served from a fresh checkout after a short first-use build; nothing else is
compiled for it.

``build()`` always compiles; ``lib()`` loads what is built and builds only
when nothing is there (guarded by a file lock so concurrent processes build
once).
"""

from __future__ import annotations

import ctypes
import fcntl
import os
import shutil
import subprocess
import tempfile
from concurrent.futures import ThreadPoolExecutor
from pathlib import Path
from typing import Optional

PKG = Path(__file__).resolve().parent.parent
CSRC = Path(__file__).resolve().parent / "csrc"
# Sources of the light library; setup.py leaves these out of the torch
# extension.
SOURCES = [
    "group_norm.hip", "xielu.hip", "mingru.hip", "attention_general.hip",
    "attention_prefill_tiles.hip", "shift_norm.hip", "latent_attention.hip", "ff_act.hip",
    "attention_latent_rows.hip", "post_norm.hip", "qkv_prep.hip", "attention_mixed_heads.hip",
    "matrix_state_scan.hip", "matrix_state_chunks.hip", "attention_mixed_heads_tiles.hip", "hyper_streams.hip",
    "routed.hip", "layer_norm.hip", "small_projection.hip", "short_conv.hip", "matrix_state_delta.hip",
]
SO_PATH = PKG / "_hybrid.so"

_LIB: Optional[ctypes.CDLL] = None


def _hipcc() -> str:
    for cand in (shutil.which("hipcc"), "/opt/rocm/bin/hipcc"):
        if cand and os.path.exists(cand):
            return cand
    raise RuntimeError("hipcc not found; cannot build the hybrid kernel library")


def build() -> Path:
    """Compile the light library for gfx950: every source on its own, side by
    side, then one link (atomic replace of the .so)."""
    workers = max(1, min(8, len(os.sched_getaffinity(0)), int(os.environ.get("MAX_JOBS") or 8)))
    flags = [
        "-O3", "-std=c++17", "--offload-arch=gfx950",
        "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops", "-fPIC",
    ]

    def run(args) -> None:
        try:
            subprocess.run([_hipcc()] + flags + args, check=True, cwd=str(CSRC),
                           stdout=subprocess.PIPE, stderr=subprocess.PIPE)
        except subprocess.CalledProcessError as e:
            raise RuntimeError(
                "building the hybrid kernel library failed:\n"
                + e.stderr.decode(errors="replace")[-4000:]
            ) from None

    with tempfile.TemporaryDirectory(prefix="._hybrid-", dir=str(PKG)) as tmp:
        objs = [os.path.join(tmp, Path(s).stem + ".o") for s in SOURCES]
        # the longest compilations first
        jobs = sorted(zip(SOURCES, objs), key=lambda j: -(CSRC / j[0]).stat().st_size)
        with ThreadPoolExecutor(max_workers=workers) as pool:
            list(pool.map(lambda j: run(["-c", str(CSRC / j[0]), "-o", j[1]]), jobs))
        so = os.path.join(tmp, "_hybrid.so")
        run(["-shared", "-o", so] + objs)
        os.chmod(so, 0o755)
        os.replace(so, SO_PATH)
    return SO_PATH


def _declare(lib: ctypes.CDLL) -> None:
    p, i, l, f = ctypes.c_void_p, ctypes.c_int, ctypes.c_long, ctypes.c_float
    sigs = {
        "lig_embed_group_norm": [p, p, p, p, f, i, i, i, i, p],
        "lig_group_norm": [p, p, p, f, i, i, i, i, p],
        "lig_post_add_pre_norm": [p, p, p, p, p, f, i, i, i, i, p],
        "lig_xielu": [p, p, f, f, l, i, p],
        "lig_sigmoid_gate_mul": [p, p, l, i, i, i, p],
        "lig_mingru_scan": [p, p, p, p, l, p, p, p, p, p, p, i, i, i, i, p],
        "lig_paged_attention_general": [
            p, p, l, p, p, p, i, p, p, p, l, p, f, f, f, i, i, i, i, i, i, i, i, i,
            i, p, i, i, f, i, p,
        ],
        "lig_offset_norm_shift": [p, p, p, p, p, p, p, p, p, p, p, p, p, p, p, f, i, i, i, p],
        "lig_offset_rms_norm": [p, p, p, f, i, i, i, p],
        "lig_residual_add": [p, p, p, l, i, p],
        "lig_latent_kv_prep": [p, p, l, p, p, p, i, p, p, p, f, i, i, i, i, i, p],
        "lig_rotate_pack_queries": [p, p, l, p, i, p, i, i, i, i, i, i, p],
        "lig_rotary_table": [p, p, p, i, i, p],
        "lig_scale_gather_rows": [p, p, p, p, l, i, i, p],
        "lig_relu_squared": [p, p, l, i, p],
        "lig_relu_squared_rows": [p, l, p, l, l, i, i, p],
        "lig_gelu_tanh_table_mul": [p, p, p, l, p, l, i, i, p],
        "lig_silu_mul": [p, p, l, i, i, p],
        "lig_kv_scatter": [p, p, l, p, p, p, i, i, i, i, i, i, p],
        "lig_temperature_scale_rows": [p, p, l, p, f, f, i, i, i, i, p],
        "lig_scaled_add_rms_norm": [p, p, p, p, p, f, f, f, f, i, i, i, p],
        "lig_qkv_norm_rope_cache": [
            p, p, p, l, p, p, p, i, p, p, f, p, p, p, f, i, i, i, i, i, i, i, i, i, i, i, p,
        ],
        "lig_token_shift_mix": [p, p, p, p, p, p, p, p, p, i, i, i, i, p],
        "lig_group_rms_norm_gate": [p, l, p, p, l, p, i, i, f, i, i, i, p],
        "lig_gelu_erf": [p, p, l, i, p],
        "lig_tanh_act": [p, p, l, i, p],
        "lig_tanh_softcap": [p, f, l, p],
        "lig_routed_combine": [p, p, p, p, p, i, p, i, i, i, i, p],
        "lig_glu_act": [p, p, l, i, i, f, f, i, p],
        "lig_residual_routed_add": [p, p, p, p, p, p, p, i, i, i, i, p],
    }
    for name, args in sigs.items():
        fn = getattr(lib, name)
        fn.argtypes = args
        fn.restype = None
    pt = lib.lig_paged_attention_prefill_tiles
    pt.argtypes = [
        p, p, l, p, p, p, l, p, p, p, p, p, p, f, f, f, i, i, i, i, i, i, i, i, i, i,
        i, p, i, i, f, p,
    ]
    pt.restype = ctypes.c_int
    hs = lib.lig_hyper_step
    hs.argtypes = [p, p, p, p, f, p, p, f, p, i, i, i, i, p]
    hs.restype = ctypes.c_int
    gr = lib.lig_grouped_topk_route
    gr.argtypes = [p, l, p, i, i, i, i, i, p, p, p]
    gr.restype = ctypes.c_int
    sp = lib.lig_small_projection
    sp.argtypes = [p, p, p, i, i, i, p]
    sp.restype = ctypes.c_int
    ln = lib.lig_layer_norm
    ln.argtypes = [p, p, p, p, f, p, p, p, f, i, i, i, p]
    ln.restype = ctypes.c_int
    mh = lib.lig_paged_attention_mixed_heads
    mh.argtypes = [p, p, l, p, p, p, i, p, p, p, i, p, f, i, i, i, i, i, i, i, i, p]
    mh.restype = ctypes.c_int
    mt = lib.lig_paged_attention_mixed_heads_tiles
    mt.argtypes = [p, p, l, p, p, p, i, p, p, p, p, p, p, f, i, i, i, i, i, i, i, i, p]
    mt.restype = ctypes.c_int
    ms = lib.lig_matrix_state_scan
    ms.argtypes = [
        p, p, l, p, l, p, l, p, p, p, p, p, l, p, p, f, p, i, f, f, p, l, p, p, p, p,
        i, i, i, i, i, i, i, p,
    ]
    ms.restype = ctypes.c_int
    lr = lib.lig_latent_attention_rows
    lr.argtypes = [p, p, p, p, p, l, p, p, p, p, i, f, i, i, i, i, i, i, i, i, p, p]
    lr.restype = ctypes.c_int
    sc = lib.lig_short_conv_silu
    sc.argtypes = [p, p, l, p, p, l, p, p, p, p, i, i, i, i, i, p]
    sc.restype = ctypes.c_int
    gd = lib.lig_gated_delta_scan
    gd.argtypes = [
        p, p, l, p, l, p, l, p, p, l, p, p, f, f, p, l, p, p, p, p, i, i, i, i, i, i, p, i, p,
    ]
    gd.restype = ctypes.c_int
    gs = lib.lig_gated_delta_scratch
    gs.argtypes = [i, i, i]
    gs.restype = l


def lib() -> ctypes.CDLL:
    global _LIB
    if _LIB is not None:
        return _LIB
    if not SO_PATH.exists():
        lock = PKG / "._hybrid.lock"
        with open(lock, "w") as lf:
            fcntl.flock(lf, fcntl.LOCK_EX)
            try:
                if not SO_PATH.exists():
                    build()
            finally:
                fcntl.flock(lf, fcntl.LOCK_UN)
    _LIB = ctypes.CDLL(str(SO_PATH))
    _declare(_LIB)
    return _LIB


def available() -> bool:
    return SO_PATH.exists()
