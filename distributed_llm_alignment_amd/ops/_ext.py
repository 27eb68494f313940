"""Loader for the in-tree gfx950 extension (`_C.so`, ops under `torch.ops.dla`).

Policy (no silent fallbacks on the GPU):
  * GPU tensors ALWAYS go through the HIP kernels. If `_C.so` is missing or fails to load and a
    GPU op is requested, `require()` raises with the build command to run.
  * CPU tensors use the pure-PyTorch reference implementations in each op module (used by the
    CPU / gloo test tier and as numerics oracles), never the other way round.
"""
from __future__ import annotations

import os
import threading
from pathlib import Path

import torch

_LOCK = threading.Lock()
_STATE = {"loaded": False, "error": None}
_GROUPS = {"core": _STATE, "mix": {"loaded": False, "error": None}}
# DLA_EXT_PATH: load an alternative build of the extension (A/B kernel experiments on one box)
SO_PATH = Path(os.environ.get("DLA_EXT_PATH") or Path(__file__).resolve().parent.parent / "_C.so")


def _so_path(group: str) -> Path:
    return SO_PATH if group == "core" else Path(__file__).resolve().parent.parent / f"_C_{group}.so"


def load(build_if_missing: bool | None = None, group: str = "core") -> bool:
    """Load a group's library once (`core`: `_C.so`, `mix`: `_C_mix.so`). Optionally build it first
    (env DLA_AUTOBUILD=1 or argument)."""
    st, path = _GROUPS[group], _so_path(group)
    with _LOCK:
        if st["loaded"]:
            return True
        if build_if_missing is None:
            build_if_missing = os.environ.get("DLA_AUTOBUILD", "0") == "1"
        try:
            if not path.exists() and build_if_missing:
                from .. import _build

                _build.build(group=group)
            if not path.exists():
                raise FileNotFoundError(str(path))
            torch.ops.load_library(str(path))
            st["loaded"] = True
            st["error"] = None
        except Exception as exc:  # surfaced by require()
            st["error"] = exc
        return st["loaded"]


def available(group: str = "core") -> bool:
    return _GROUPS[group]["loaded"] or load(group=group)


def require(group: str = "core"):
    """Return the op namespace or raise loudly (GPU path must never fall back silently)."""
    if not available(group):
        raise RuntimeError(
            f"distributed_llm_alignment_amd HIP extension ({group} group) is not loaded "
            f"({_GROUPS[group]['error']!r}). Build it with: "
            "DLA_SKIP_EXT_LOAD=1 python -m distributed_llm_alignment_amd._build"
        )
    return torch.ops.dla


def use_native(*tensors: torch.Tensor) -> bool:
    """True when the op must run on the HIP kernels (any operand on the GPU)."""
    for t in tensors:
        if isinstance(t, torch.Tensor) and t.is_cuda:
            return True
    return False
