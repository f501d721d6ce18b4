"""Trace replay: feeds given tokens through a model step by step and writes
logits, on the engine's own step function (Engine.execute), cache and state
manager, and kernels. Nothing is sampled.

Steps are JSON objects, one a line, on standard input:

  {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}],
   "end": ["b"]}

An entry brings a request's next tokens; `want` are places among them whose
logits are written to OUT/<step>.f32 (float32, little-endian, entries in
order). `end` names requests whose pages and slots are given back after the
step. After each step the line "done <step>" is printed.
"""

from __future__ import annotations

import argparse
import fcntl
import json
import os
import subprocess
import sys
from typing import TextIO

ROOT = os.path.dirname(os.path.dirname(os.path.dirname(
    os.path.abspath(__file__))))
MAX_REQUESTS = 4        # state slots


def ensure_built() -> None:
    """Compile the kernels of hybrid models in place if they are not there
    (fresh checkout); concurrent first calls wait for one another."""
    import torch  # noqa: F401  (its libraries must be loaded first)

    def built() -> bool:
        import importlib
        importlib.invalidate_caches()
        try:
            importlib.import_module("substratus_amd._hybrid")
            return True
        except ImportError:
            return False

    if built():
        return
    with open(os.path.join(ROOT, ".build.lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if not built():
            subprocess.run(
                [sys.executable, "setup.py", "build_ext", "--inplace"],
                cwd=ROOT, check=True, stdout=sys.stderr,
                env=dict(os.environ, PYTORCH_ROCM_ARCH="gfx950",
                         SUB_EXT="_hybrid"))
            if not built():   # imports it afresh, past the import cache
                raise RuntimeError("built, but cannot be imported: "
                                   "substratus_amd._hybrid")


class TraceReplay:
    def __init__(self, model_dir: str, dtype: str, max_tokens: int,
                 device: str = "cuda"):
        import torch

        from ..models.weights import load_weights
        from .engine import Engine, EngineConfig
        from .kv_cache import DEFAULT_BLOCK_SIZE
        # float32 means float32, whatever the process's defaults are
        torch.set_float32_matmul_precision("highest")
        blocks = -(-max_tokens // DEFAULT_BLOCK_SIZE)
        self.engine = Engine(EngineConfig(
            model=model_dir, dtype=getattr(torch, dtype),
            max_batch=MAX_REQUESTS, max_seq_len=blocks * DEFAULT_BLOCK_SIZE,
            kv_blocks=blocks), device=device)
        if not self.engine.takes_portions:
            raise ValueError(f"{self.engine.mcfg.family} models do not take "
                             "portions of prompts")
        if not load_weights(self.engine.model, self.engine.mcfg, model_dir,
                            self.engine.device, self.engine.cfg.dtype):
            raise FileNotFoundError(f"no weights in {model_dir}")
        self.live: dict = {}

    def step(self, entries: list[dict], end: list[str]):
        """Logits of the wanted places, float32 on the host [wanted, vocab]."""
        from .kv_cache import SequenceState
        work = []
        for e in entries:
            seq = self.live.get(e["id"])
            if seq is None:
                seq = self.live[e["id"]] = SequenceState(
                    seq_id=len(self.live), tokens=[], num_prompt=0,
                    max_new_tokens=0)
            if not e["tokens"]:
                continue
            seq.tokens.extend(e["tokens"])
            if seq.length > self.engine.cfg.max_seq_len:
                raise ValueError(f"request {e['id']} is longer than "
                                 f"{self.engine.cfg.max_seq_len} tokens")
            self.engine.kv.reserve(seq, seq.length)
            work.append((seq, len(e["tokens"]), e["want"]))
        logits = self.engine.execute(work).float().cpu() if work else None
        for name in end:
            if name in self.live:
                self.engine.kv.release(self.live.pop(name))
        return logits


def replay(trace: TraceReplay, steps: TextIO, out_dir: str) -> None:
    for line in steps:
        if not line.strip():
            continue
        doc = json.loads(line)
        logits = trace.step(doc["entries"], doc.get("end", []))
        if any(e["want"] for e in doc["entries"]):
            path = os.path.join(out_dir, f"{doc['step']}.f32")
            logits.numpy().astype("<f4").tofile(path)
        print(f"done {doc['step']}", flush=True)


def main(argv: list[str] | None = None) -> int:
    p = argparse.ArgumentParser(
        prog="trace_run", description="Replay a trace of tokens and write "
        "logits; steps come as JSON lines on standard input.")
    p.add_argument("--model", required=True, metavar="DIR",
                   help="folder with config.json and model.safetensors")
    p.add_argument("--dtype", choices=["bfloat16", "float32"],
                   default="bfloat16")
    p.add_argument("--out", required=True, metavar="DIR",
                   help="where <step>.f32 files go")
    p.add_argument("--max-tokens", type=int, required=True,
                   help="size of the cache pool in tokens")
    p.add_argument("--device", default="cuda",
                   help="cuda, or cpu for the plain reference ops")
    a = p.parse_args(argv)
    if a.device != "cpu":
        ensure_built()
    trace = TraceReplay(a.model, a.dtype, a.max_tokens, a.device)
    replay(trace, sys.stdin, a.out)
    return 0


if __name__ == "__main__":
    sys.exit(main())
