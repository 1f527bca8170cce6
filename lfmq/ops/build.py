"""Build an in-tree HIP extension on first use.

A fresh checkout holds sources only.  Entry points that must work there
(bin/trace_run) compile the one extension that they need; a lock file
keeps two first calls from building at once.
"""
from __future__ import annotations

import fcntl
import glob
import os
import subprocess
import sys

REPO = os.path.dirname(os.path.dirname(os.path.dirname(os.path.abspath(__file__))))


def built(name: str) -> bool:
    return bool(glob.glob(os.path.join(REPO, f"{name}*.so")))


def ensure_built(name: str) -> None:
    """Compile extension `name` into the checkout unless it is there."""
    if built(name):
        return
    with open(os.path.join(REPO, f".build-{name}.lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if built(name):
            return
        env = dict(os.environ, PYTORCH_ROCM_ARCH="gfx950",
                   LFMQ_EXTENSIONS=name)
        r = subprocess.run([sys.executable, "setup.py", "build_ext",
                            "--inplace"], cwd=REPO, env=env,
                           stdin=subprocess.DEVNULL, stdout=subprocess.PIPE,
                           stderr=subprocess.STDOUT, text=True)
        if r.returncode:
            sys.stderr.write(r.stdout[-8000:])
            raise RuntimeError(f"building {name} failed ({r.returncode})")
