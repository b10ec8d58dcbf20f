"""Replay of given tokens through the engine, step by step: ``bin/trace_run``.

A step is one batch of portions of prompts and single tokens, each from a request that may come and go; what is asked for
are the logits at given places.  Nothing is sampled.  The model, the loader, the block pool, the batch builder, the
executor and its KV cache are the ones that serve generation (``ModelRunner``); only the scheduler's decisions and the
token values come from outside."""
from __future__ import annotations

import argparse
import json
import os
import sys

import torch

from ..config import Config
from .block_manager import BlockManager
from .model_runner import ModelRunner
from .sequence import Sequence

__all__ = ["StepReplayer", "main"]

MAX_LIVE = 4   # requests live at any time


class StepReplayer:
    def __init__(self, model: str, dtype: str, max_tokens: int, max_live: int = MAX_LIVE, block_size: int = 64,
                 runner=None) -> None:
        blocks = -(-max_tokens // block_size)
        self.config = Config(model, dtype=dtype, kvcache_block_size=block_size, num_kvcache_blocks=blocks,
                             max_num_seqs=max_live, max_model_len=blocks * block_size,
                             max_num_batched_tokens=blocks * block_size, enforce_eager=True)
        self.runner = runner if runner is not None else ModelRunner(self.config, 0)
        self.blocks = BlockManager(blocks, block_size,
                                   state_slots=max_live if getattr(self.config.hf_config, "recurrent_state", False) else 0)
        self.live: dict[str, Sequence] = {}
        self.vocab = self.config.hf_config.vocab_size

    def step(self, entries: list[dict], end: list[str] = ()) -> torch.Tensor | None:
        """-> logits [wanted, vocab] in fp32 on the host, or None when nothing is wanted."""
        if len({e["id"] for e in entries}) != len(entries):
            raise ValueError("a request appears twice in one step")
        seqs, rows = [], []
        for e in entries:
            tokens, want = [int(t) for t in e["tokens"]], [int(w) for w in e.get("want", [])]
            if not tokens or not all(0 <= t < self.vocab for t in tokens):
                raise ValueError(f"request {e['id']}: token ids must be in [0, {self.vocab})")
            if not all(0 <= w < len(tokens) for w in want):
                raise ValueError(f"request {e['id']}: wanted places must be in [0, {len(tokens)})")
            seq = self.live.get(e["id"])
            if seq is None:
                if len(self.live) >= self.config.max_num_seqs:
                    raise ValueError(f"more than {self.config.max_num_seqs} live requests")
                seq = self.live[e["id"]] = Sequence(tokens, block_size=self.blocks.block_size)
            else:
                seq.extend(tokens)
            self.blocks.reserve(seq)
            seqs.append(seq)
            rows.append(want)
        logits = self.runner.inference_executor.score_batch(seqs, rows) if seqs else None
        out = None if logits is None else logits.float().cpu()
        torch.cuda.synchronize()          # the staging buffers of this step may be refilled by the next
        for name in end:
            self.blocks.deallocate(self.live.pop(name))
        return out

    def close(self) -> None:
        self.runner.exit()


def main(argv: list[str] | None = None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay steps of token ids (standard input, one JSON object "
                                 "each) through a model and write the logits asked for.")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], required=True)
    ap.add_argument("--out", required=True, help="folder for <step>.f32 (little-endian floats, [wanted, vocab])")
    ap.add_argument("--max-tokens", type=int, required=True, help="tokens that live requests hold at most")
    a = ap.parse_args(argv)
    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")
    os.makedirs(a.out, exist_ok=True)
    replayer = StepReplayer(a.model, a.dtype, a.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = replayer.step(step["entries"], step.get("end", []))
        if logits is not None:
            logits.contiguous().numpy().astype("<f4", copy=False).tofile(os.path.join(a.out, f"{step['step']}.f32"))
        print(f"done {step['step']}", flush=True)
    replayer.close()
    return 0
