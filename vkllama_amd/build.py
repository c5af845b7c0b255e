"""Compiles the two product libraries in place (a checkout holds sources only)."""
import fcntl
import os
import subprocess
import sys

_PKG = os.path.dirname(os.path.abspath(__file__))
LIBS = ("libvkllama_hip.so", "libvkllama_host.so")


def ensure_built(jobs=None):
    """Builds libvkllama_hip.so and libvkllama_host.so unless both are there.
    Safe to call from several processes at once; the compilers' output goes to
    standard error."""
    lib = os.path.join(_PKG, "lib")

    def missing():
        return [n for n in LIBS if not os.path.exists(os.path.join(lib, n))]
    if not missing():
        return
    jobs = str(jobs or min(16, os.cpu_count() or 1))
    os.makedirs(lib, exist_ok=True)
    with open(os.path.join(lib, ".lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if missing():
            for args in (["-C", os.path.join(_PKG, "csrc")], ["-C", os.path.join(_PKG, "host"), "lib"]):
                subprocess.run(["make", "-j" + jobs] + args, check=True, stdin=subprocess.DEVNULL, stdout=sys.stderr)
