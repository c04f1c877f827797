"""Builds the native library where it is missing: the bf16-weight part alone (``make models``), which is all that a model
with bf16 weights needs.  Uses nothing but the standard library, so that it can run before the package is imported."""
from __future__ import annotations

import fcntl
import os
import subprocess
import sys

_HERE = os.path.dirname(os.path.abspath(__file__))


def ensure_built() -> None:
    """Returns at once when ``liblocal_hip.so`` or its bf16-weight part is there; otherwise compiles the latter.  The
    compiler's output goes to standard error; of several processes one builds and the others wait."""
    names = ("liblocal_hip.so", "liblocal_hip_models.so")
    if any(os.path.exists(os.path.join(_HERE, n)) for n in names):
        return
    build = os.path.join(_HERE, "csrc", "build")
    os.makedirs(build, exist_ok=True)
    with open(os.path.join(build, ".lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if any(os.path.exists(os.path.join(_HERE, n)) for n in names):
            return
        part = os.path.join(_HERE, f".models-{os.getpid()}.so")     # renamed when complete: nobody loads half a library
        jobs = str(min(16, os.cpu_count() or 4))
        subprocess.run(["make", "-C", os.path.join(_HERE, "csrc"), "-j", jobs, "models", f"MODELS_OUT={part}"], check=True,
                       stdout=sys.stderr)
        os.replace(part, os.path.join(_HERE, names[1]))
