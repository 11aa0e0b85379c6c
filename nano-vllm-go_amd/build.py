"""Compiles csrc/ into lib/libnvllm_hip.so for gfx950 (hipcc cross-compiles without a GPU)."""
from __future__ import annotations

import os
import subprocess
from pathlib import Path

_PKG = Path(__file__).resolve().parent


def build(force: bool = False) -> Path:
    jobs = min(int(os.environ.get("MAX_JOBS") or 16), os.cpu_count() or 1, 16)
    args = ["make", "-C", str(_PKG / "csrc"), "-s", f"-j{jobs}"]
    if force:
        args.append("-B")
    subprocess.check_call(args)
    out = _PKG / "lib" / "libnvllm_hip.so"
    assert out.exists(), out
    return out


if __name__ == "__main__":
    print(build())
