"""Build the HIP extensions that are missing, in-tree.

setup.py runs in a child process of its own; a lock keeps two callers from
building into the same tree at once."""
from __future__ import annotations

import fcntl
import glob
import os
import subprocess
import sys

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _missing(names):
    return [n for n in names
            if not glob.glob(os.path.join(ROOT, "nanorlhf_amd", f"{n}.*.so"))]


def ensure_built(names) -> None:
    """Compile those of the extensions `names` that are not built yet.  The
    compiler's output goes to standard error."""
    if not _missing(names):
        return
    os.makedirs(os.path.join(ROOT, "build"), exist_ok=True)
    with open(os.path.join(ROOT, "build", ".lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        todo = _missing(names)
        if todo:
            env = dict(os.environ, NANORLHF_EXT=",".join(todo), PYTORCH_ROCM_ARCH="gfx950")
            subprocess.run([sys.executable, "setup.py", "build_ext", "--inplace"], cwd=ROOT,
                           env=env, check=True, stdout=sys.stderr.fileno())
