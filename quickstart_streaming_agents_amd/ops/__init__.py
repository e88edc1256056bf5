"""Op layer: the hand-written HIP/CDNA4 kernels + CPU references.

Two native modules: qsa_hip (streaming, retrieval, Llama/Mixtral/encoder
kernels) and qsa_lm_hip (mixer decoders: retention, latent and grouped-query
attention, short convolutions, state-space duality, f32 residual norms, greedy
pick).

Fail-loud contract: on a GPU box the HIP extension MUST be importable —
there is no silent eager fallback for the hot ops.  CPU-only environments
(unit tests, this dev container) use ops.cpu_ref directly and never touch
the extension.
"""

from __future__ import annotations

_ext = None
_import_error: Exception | None = None
try:
    import torch  # noqa: F401  (loads libc10/libtorch the extension links)
    from .. import qsa_hip as _ext  # built in-tree by setup.py
except ImportError as e:  # pragma: no cover - exercised only when unbuilt
    _import_error = e

_lm_ext = None
_lm_import_error: Exception | None = None
try:
    from .. import qsa_lm_hip as _lm_ext
except ImportError as e:  # pragma: no cover - exercised only when unbuilt
    _lm_import_error = e


def have_lm_ext() -> bool:
    return _lm_ext is not None


def lm_ext():
    """The qsa_lm_hip module; raises loudly if the native build is missing."""
    if _lm_ext is None:
        raise RuntimeError(
            "qsa_lm_hip extension not built. Run "
            "`python setup.py build_ext --inplace` "
            f"(import error: {_lm_import_error})")
    return _lm_ext


def have_ext() -> bool:
    return _ext is not None


def ext():
    """The qsa_hip module; raises loudly if the native build is missing."""
    if _ext is None:
        raise RuntimeError(
            "qsa_hip extension not built. Run "
            "`python setup.py build_ext --inplace` "
            f"(import error: {_import_error})")
    return _ext
