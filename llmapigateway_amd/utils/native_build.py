"""Compiling the in-tree HIP extensions (setup.py) when they are missing."""

from __future__ import annotations

import fcntl
import glob
import os
import subprocess
import sys
from typing import Sequence

ROOT = os.path.dirname(os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
EXTENSIONS = ("_C", "_H")


def is_built(name: str) -> bool:
    return bool(glob.glob(os.path.join(ROOT, "llmapigateway_amd", "ops", f"{name}.*.so")))


def build(names: Sequence[str] = EXTENSIONS) -> None:
    """Compile these extensions for gfx950, in-tree; compiler output goes to
    stderr."""
    subprocess.run(
        [sys.executable, "setup.py", "build_ext", "--inplace"],
        cwd=ROOT,
        env=dict(os.environ, PYTORCH_ROCM_ARCH="gfx950", LLMAPI_EXT=",".join(names)),
        stdout=sys.stderr,
        check=True,
    )


def ensure_built(name: str) -> None:
    """Compile one extension if nothing of it is there (one process builds,
    others wait)."""
    if is_built(name):
        return
    os.makedirs(os.path.join(ROOT, "build"), exist_ok=True)
    with open(os.path.join(ROOT, "build", ".lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if not is_built(name):
            build([name])
