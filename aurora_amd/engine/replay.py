"""Trace replay: given token ids through the engine, logits out.

A trace is a list of steps; a step brings the next tokens of some requests
(portions of prompts beside single tokens), all of which run as one batch, and
names the requests that end after it. Nothing is sampled or scheduled: the
trace says what runs, and the engine's own reservation, batch building,
forward, decode graphs and cache managers run it.

    bin/trace_run --model DIR --dtype bfloat16 --out DIR --max-tokens N < steps
"""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, List, Optional, Sequence as Seq, Tuple

import torch

from .engine import EngineConfig, LLMEngine, Sequence
from .sampling_params import SamplingParams


class TraceReplayer:
    def __init__(self, engine: LLMEngine):
        self.engine = engine
        self.live: Dict[str, Sequence] = {}

    def step(self, entries: Seq[Tuple[str, List[int], List[int]]],
             end: Seq[str] = ()) -> Optional[torch.Tensor]:
        """Run (id, next tokens, wanted places among them) entries as one
        batch; logits of the wanted places in order, None if there are none."""
        eng = self.engine
        prefill: List[Tuple[Sequence, int, List[int]]] = []
        decode: List[Tuple[Sequence, List[int]]] = []
        order = []  # (is_prefill, index) of each entry
        for rid, tokens, want in entries:
            if not tokens:
                raise ValueError(f"request {rid}: an entry without tokens")
            vocab = eng.spec.vocab_size
            if min(tokens) < 0 or max(tokens) >= vocab:
                raise ValueError(f"request {rid}: token id outside [0, {vocab})")
            seq = self.live.get(rid)
            if seq is None:
                seq = Sequence(rid, [], SamplingParams())
                self.live[rid] = seq
            seq.token_ids.extend(tokens)
            if seq.num_tokens > eng.max_model_len:
                raise ValueError(f"request {rid} is longer than {eng.max_model_len} tokens")
            if not eng._try_reserve(seq, seq.num_tokens):
                raise MemoryError(f"no cache pages or state slot left for request {rid}")
            if seq.num_cached and len(tokens) == 1:
                order.append((False, len(decode)))
                decode.append((seq, want))
            else:
                order.append((True, len(prefill)))
                prefill.append((seq, len(tokens), want))
        first = [0]
        for _, n, _ in prefill:
            first.append(first[-1] + n)
        rows: List[int] = []
        for is_prefill, i in order:
            if is_prefill:
                rows.extend(first[i] + w for w in prefill[i][2])
            else:
                rows.extend(first[-1] + i for _ in decode[i][1])
        logits = None
        if prefill or decode:
            logits = eng.execute([p[0] for p in prefill], [p[1] for p in prefill],
                                 [d[0] for d in decode], rows)
        for rid in end:
            eng._release(self.live.pop(rid))
        return logits


def make_engine(model: str, dtype: str, max_tokens: int, device: str = "auto",
                max_requests: int = 4, page_size: int = 64) -> LLMEngine:
    """An engine whose pool holds ``max_tokens`` tokens and whose recurrent
    state has ``max_requests`` slots."""
    pages = -(-max_tokens // page_size)
    graphs = device != "cpu" and torch.cuda.is_available()
    return LLMEngine(EngineConfig(
        model=model, dtype=dtype, device=device, page_size=page_size,
        # one more page takes the writes of idle rows of captured batches
        kv_cache_pages=pages + (1 if graphs else 0),
        max_num_seqs=max_requests, state_slots=max_requests,
        max_model_len=pages * page_size, use_hip_graphs=graphs))


def main(argv: Optional[List[str]] = None) -> int:
    ap = argparse.ArgumentParser(
        prog="trace_run", description="Replay a trace of token ids (JSON lines "
        "on standard input) through a model and write the wanted logits.")
    ap.add_argument("--model", required=True,
                    help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for <step>.f32 files")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="capacity of the cache pool in tokens, over all unfinished requests")
    ap.add_argument("--device", choices=("auto", "cpu"), default="auto")
    args = ap.parse_args(argv)
    if args.device == "auto" and not torch.cuda.is_available():
        print("trace_run: no GPU (use --device cpu for the reference ops)",
              file=sys.stderr)
        return 1
    replayer = TraceReplayer(make_engine(args.model, args.dtype, args.max_tokens,
                                         args.device))
    os.makedirs(args.out, exist_ok=True)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = replayer.step(
            [(e["id"], e["tokens"], e.get("want", [])) for e in step.get("entries", [])],
            step.get("end", ()))
        if logits is not None:
            with open(os.path.join(args.out, f"{step['step']}.f32"), "wb") as f:
                f.write(logits.float().cpu().numpy().astype("<f4").tobytes())
        print(f"done {step['step']}", flush=True)
    return 0
