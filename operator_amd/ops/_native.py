"""Loader for the in-tree native extensions.

The gfx950 kernel modules (``operator_amd._C``: the language models; ``operator_amd._S``: log
scan, scoring, collectives) are REQUIRED whenever a GPU tensor reaches an op: there is no
silent eager fallback on the device. Each is loaded, and built if need be, at its first use. CPU tensors use
the plain-PyTorch reference implementations (operator_amd.ops.reference), which
exist for the CPU test tier and for numerics checks of the HIP kernels.
"""
from __future__ import annotations

import importlib
import os
import threading

import torch  # noqa: F401  (must be imported before _C: one HIP runtime per process)

_lock = threading.RLock()
_C = None
_S = None
_P = None


def _try_build(name: str) -> None:
    if os.environ.get("OAMD_NO_AUTOBUILD"):
        return
    from operator_amd import _build

    _build.build_kernels(modules=(name,))


def _check_fresh(mod_name: str, srcs: list[str]) -> None:
    """Refuse an in-tree extension older than any of its sources: a GPU run of stale
    kernels (e.g. a host-side contract the old binary does not implement) can fault the
    device. OAMD_ALLOW_STALE=1 skips the check."""
    if os.environ.get("OAMD_ALLOW_STALE"):
        return
    import glob

    root = os.path.dirname(os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
    so = glob.glob(os.path.join(root, "operator_amd", mod_name + ".*.so"))
    if not so:
        return
    built = min(os.path.getmtime(f) for f in so)
    newer = [os.path.relpath(f, root) for f in srcs if os.path.getmtime(f) > built + 1.0]
    if newer:
        raise RuntimeError(f"operator_amd.{mod_name} is older than {newer[:4]}: rebuild with "
                           "`python -m operator_amd._build` (or set OAMD_ALLOW_STALE=1)")


def _sources(name: str) -> list[str]:
    from operator_amd import _build

    if name == "_patterns":
        return [str(f) for f in (_build.CSRC / "patterns").glob("*")]
    return [str(f) for f in _build.module_sources(name) + sorted((_build.CSRC / "kernels").glob("*.h"))]


def _load(name: str):
    """Import native kernel module ``name``, building it in-tree if it is not there."""
    _check_fresh(name, _sources(name))
    try:
        return importlib.import_module("operator_amd." + name)
    except ImportError as e:  # not built yet
        try:
            _try_build(name)
            return importlib.import_module("operator_amd." + name)
        except Exception as e2:  # pragma: no cover - exercised only without hipcc
            raise RuntimeError(f"operator_amd.{name} (gfx950 kernels) unavailable: {e2}") from e


class _Kernels:
    """Both kernel modules as one namespace: names of ``_C`` first; the first name it does not
    have brings in ``_S``. Resolved names are kept as instance attributes."""

    def __init__(self, c):
        self._c = c

    def __getattr__(self, name: str):
        if name.startswith("__"):
            raise AttributeError(name)
        mod = self._c if hasattr(self._c, name) else _services()
        v = getattr(mod, name)
        setattr(self, name, v)
        return v


def _services():
    global _S
    with _lock:
        if _S is None:
            _S = _load("_S")
    return _S


def kernels():
    """The compiled gfx950 kernels (building what is missing in-tree)."""
    global _C
    if _C is None:
        with _lock:
            if _C is None:
                _C = _Kernels(_load("_C"))
    return _C


def patterns():
    """Return the CPU pattern compiler / packer / scorer module."""
    global _P
    if _P is not None:
        return _P
    with _lock:
        if _P is None:
            _check_fresh("_patterns", _sources("_patterns"))
            try:
                _P = importlib.import_module("operator_amd._patterns")
            except ImportError:
                from operator_amd import _build

                _build.build_patterns()
                _P = importlib.import_module("operator_amd._patterns")
    return _P


def native_available() -> bool:
    try:
        kernels()
        return True
    except Exception:
        return False
