"""Compiles libmagicdec_hip.so from csrc/ (hipcc, gfx950)."""
from __future__ import annotations

import os
import subprocess
import sys

_HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(_HERE, "csrc")
LIB = os.path.join(_HERE, "libmagicdec_hip.so")


def build_library(force=False, stdout=None):
    """Runs the Makefile (force: every object anew)."""
    jobs = min(int(os.environ.get("MAX_JOBS") or os.cpu_count() or 4), 16)
    subprocess.run(["make", "-C", CSRC, f"-j{jobs}"] + (["-B"] if force else []), check=True, stdout=stdout)


def ensure_built():
    """The library of a fresh checkout; a built one is taken as it is."""
    if not os.path.exists(LIB):
        print("[magicdec_amd] compiling libmagicdec_hip.so", file=sys.stderr, flush=True)
        build_library(stdout=sys.stderr)
