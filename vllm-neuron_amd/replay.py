# SPDX-License-Identifier: Apache-2.0
"""Trace replay: given token ids through the engine step by step, logits out (bin/trace_run).

Every step is one engine step: the scheduler admits and schedules the requests, its block pool hands out KV blocks, the
runner builds the ragged batch, the library runs it; nothing is sampled.

    trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N      < steps (JSON lines)

A step: {"step": n, "entries": [{"id", "tokens", "want"}], "end": [ids]}.  Where something is wanted DIR/<n>.f32 holds
the logits [wanted, vocab] in the order of the entries; every step is answered by a line "done <n>"."""

from __future__ import annotations

import argparse
import json
import os
import sys

BLOCK_SIZE = 32        # divides the 64 tokens a request's count is rounded up to
MAX_LIVE_REQUESTS = 4


class TraceReplay:
    """`engine`: a chunked-prefill MI355XEngine without prefix caching (every token brought is computed)."""

    def __init__(self, engine):
        self.engine = engine
        self.live: set = set()

    @classmethod
    def from_dir(cls, model_dir: str, dtype: str, max_tokens: int, max_live: int = MAX_LIVE_REQUESTS):
        from .models import load_config
        return cls.from_config(load_config(model_dir), dtype, max_tokens, max_live, model=model_dir)

    @classmethod
    def from_config(cls, config, dtype: str, max_tokens: int, max_live: int = MAX_LIVE_REQUESTS, block_size: int = BLOCK_SIZE,
                    model: str = "", override: dict | None = None):
        from .engine import MI355XEngine
        return cls(MI355XEngine(
            config, model, dtype=dtype, max_model_len=min(config.max_position_embeddings, max_tokens), max_num_seqs=max_live,
            block_size=block_size, num_gpu_blocks_override=-(-max_tokens // block_size), enable_prefix_caching=False,
            enable_chunked_prefill=True, max_num_batched_tokens=max_tokens,
            override_mi355x_config={"is_block_kv_layout": True, "weight_artifacts": False, "kv_overcommit": True,
                                    "chunked_prefill_config": {"max_num_seqs": max_live}, **(override or {})}))

    def step(self, entries: list, end: list):
        """-> the wanted logits, one [len(want), vocab] tensor per entry"""
        from ._vllm_compat import SamplingParams
        for e in entries:
            if e["id"] in self.live:
                self.engine.append_tokens(e["id"], e["tokens"])
            else:
                self.engine.add_request(list(e["tokens"]), SamplingParams(temperature=0.0, max_tokens=1), request_id=e["id"])
                self.live.add(e["id"])
        logits, sched = self.engine.score_step({e["id"]: e.get("want") or [] for e in entries})
        for e in entries:
            got = sched.num_scheduled_tokens.get(e["id"], 0)
            if got != len(e["tokens"]):
                raise RuntimeError(f"request {e['id']}: {got} of {len(e['tokens'])} tokens scheduled (KV pool or request slots exhausted)")
        if end:
            self.engine.finish_requests(list(end))
            self.live.difference_update(end)
        return [logits[e["id"]] for e in entries]


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a token trace through the engine and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for <step>.f32 files")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens live requests hold at any time (sizes the KV pool)")
    args = ap.parse_args(argv)
    replay = TraceReplay.from_dir(args.model, args.dtype, args.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        wanted = [t for t in replay.step(step["entries"], step.get("end") or []) if t.shape[0]]
        if wanted:
            path = os.path.join(args.out, f"{step['step']}.f32")
            with open(path, "wb") as f:
                for t in wanted:
                    f.write(t.contiguous().numpy().astype("<f4", copy=False).tobytes())
        print(f"done {step['step']}", flush=True)
    replay.engine.close()
    return 0
