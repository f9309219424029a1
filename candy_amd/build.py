"""Compiling libcandy_hip.so where a checkout does not hold it yet."""
from __future__ import annotations

import fcntl
import os
import subprocess
import sys

from . import hip

CSRC = os.path.join(os.path.dirname(os.path.abspath(__file__)), "csrc")


def ensure_library() -> None:
    """Builds the library unless it is there; concurrent callers wait for one build."""
    if os.path.exists(hip.LIB_PATH):
        return
    with open(os.path.join(CSRC, ".build.lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if os.path.exists(hip.LIB_PATH):
            return
        jobs = os.environ.get("MAX_JOBS") or str(min(16, os.cpu_count() or 1))
        subprocess.run(["make", "-C", CSRC, "-j" + jobs], check=True, stdin=subprocess.DEVNULL, stdout=sys.stderr)
