"""Building libmuillm_amd.so from the sources of a checkout (hipcc, gfx950)."""
import fcntl
import os
import subprocess
import sys

_CSRC = os.path.join(os.path.dirname(os.path.abspath(__file__)), "csrc")


def make(force: bool = False, log=None) -> None:
    jobs = min(16, int(os.environ.get("MAX_JOBS") or os.cpu_count() or 1))
    subprocess.run(["make", "-C", _CSRC, "-j", str(max(1, jobs))] + (["-B"] if force else []), check=True, stdout=log)


def ensure_built() -> None:
    """Build the library if it is not there (one process at a time; the others wait and use the result)."""
    from . import _lib

    if os.path.exists(_lib.LIB_PATH):
        return
    with open(os.path.join(_CSRC, ".build.lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if not os.path.exists(_lib.LIB_PATH):
            make(log=sys.stderr)
