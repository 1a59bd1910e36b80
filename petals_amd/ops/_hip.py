"""Loader for the in-tree HIP extensions (.so files built by petals_amd.ops.build)."""

from __future__ import annotations

import importlib.util
import os

from petals_amd.ops.build import EXTENSIONS, so_path


_loaded = {}


def first_loaded(*names: str):
    """The first of these libraries that this process has loaded; if it has
    loaded none, the first that is built."""
    for name in names:
        if name in _loaded:
            return _loaded[name]
    name = next((n for n in names if os.path.exists(so_path(n))), names[0])
    _loaded[name] = load(name)
    return _loaded[name]


def load(name: str = "core"):
    import torch  # noqa: F401 — the extension links against loaded libtorch

    path = so_path(name)
    if not os.path.exists(path):
        raise ImportError(f"HIP extension not built: {path} missing (run python -m petals_amd.ops.build)")
    spec = importlib.util.spec_from_file_location(EXTENSIONS[name][1], path)
    module = importlib.util.module_from_spec(spec)
    spec.loader.exec_module(module)
    return module
