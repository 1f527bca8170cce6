"""Op bindings: the single compute backend is PyTorch-ROCm + the in-tree
HIP extensions (csrc/ -> lfmq_hip.so and lfmq_seq.so, gfx950 only).

There is deliberately NO multi-backend dispatch:
on a GPU device the HIP extension is the only path and a missing extension
raises immediately instead of silently falling back to eager PyTorch.  The
CPU twins in lfmq.ops.ref exist for unit tests and for the OPT-125m int8
CPU decode config, which is spec'd as a CPU path.
"""
from __future__ import annotations

from . import ref  # noqa: F401

_EXTS: dict = {}       # name -> module, or the import error's text


def _load_ext(name: str = "lfmq_hip"):
    if name not in _EXTS:
        try:
            import importlib
            _EXTS[name] = importlib.import_module(name)
        except Exception as e:  # pragma: no cover - only without the .so
            _EXTS[name] = f"{type(e).__name__}: {e}"
    return None if isinstance(_EXTS[name], str) else _EXTS[name]


def _require(name: str):
    ext = _load_ext(name)
    if ext is None:
        raise RuntimeError(
            f"{name} extension not built (run `python setup.py build_ext "
            f"--inplace`, PYTORCH_ROCM_ARCH=gfx950). Import error: "
            f"{_EXTS[name]}")
    return ext


def hip_ext():
    """The loaded HIP extension module, or raise.  GPU code MUST go through
    this — never fall back to eager torch on a GPU device."""
    return _require("lfmq_hip")


def seq_ext():
    """The extension of the sequence-mixing layers and of the small ops
    that every model shares, or raise."""
    return _require("lfmq_seq")


def hip_ext_available() -> bool:
    return _load_ext() is not None
