"""Trace replay over the batch engine (`bin/trace_run`)."""

from __future__ import annotations

import argparse
import fcntl
import importlib.util
import json
import os
import subprocess
import sys
from pathlib import Path

ROOT = Path(__file__).resolve().parents[2]
MAX_REQUESTS = 4


def build_kernels():
    """Compile the extension the batch engine's models load, if it is not
    there; concurrent calls wait for the first."""
    def importable() -> bool:
        importlib.invalidate_caches()
        return importlib.util.find_spec("mlx_sharding_amd._hip_ragged") is not None

    if importable():
        return
    with open(ROOT / ".build_lock", "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if importable():
            return
        env = dict(os.environ, MLXS_AMD_EXT="_hip_ragged")
        env.setdefault("MAX_JOBS", "8")
        subprocess.run([sys.executable, "setup.py", "build_ext", "--inplace"],
                       cwd=ROOT, env=env, check=True, stdout=sys.stderr)


def parse_args(argv=None):
    p = argparse.ArgumentParser(description=__doc__)
    p.add_argument("--model", required=True)
    p.add_argument("--dtype", required=True, choices=["bfloat16", "float32"])
    p.add_argument("--out", required=True)
    p.add_argument("--max-tokens", type=int, required=True,
                   help="most tokens that live requests hold at any time, "
                        "each rounded up to whole cache pages")
    p.add_argument("--device", default="cuda")
    return p.parse_args(argv)


def main(argv=None) -> int:
    args = parse_args(argv)
    import torch

    if args.device.startswith("cuda"):
        build_kernels()

    from ..parallel.batching import BatchEngine, Portion
    from ..utils.loading import load_model

    model, _ = load_model(args.model, device=args.device,
                          dtype=getattr(torch, args.dtype))
    engine = BatchEngine(model, args.max_tokens, MAX_REQUESTS)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        portions = [Portion(e["id"], e["tokens"], e.get("want") or ())
                    for e in step["entries"]]
        logits = engine.step(portions)
        if logits.shape[0]:
            data = logits.float().cpu().contiguous().numpy().astype("<f4")
            with open(os.path.join(args.out, f"{step['step']}.f32"), "wb") as f:
                f.write(data.tobytes())
        for rid in step.get("end") or ():
            engine.end(rid)
        print(f"done {step['step']}", flush=True)
    return 0
