# SPDX-License-Identifier: Apache-2.0
"""Command line of the standalone engine: token-id prompts in, generated token ids out (bin/generate).

    generate --model DIR --prompt 1,2,3 --prompt 9,8,7,6 --max-tokens 32

config.json picks the model (models/__init__.py); one JSON line per prompt."""

from __future__ import annotations

import argparse
import json


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="generate", description="generate from token-id prompts")
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--prompt", action="append", required=True, metavar="IDS", help="comma-separated token ids (repeatable)")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16",
                    help="float32: layer-stack models only (32-bit compute, for checking)")
    ap.add_argument("--max-tokens", type=int, default=16)
    ap.add_argument("--temperature", type=float, default=0.0)
    ap.add_argument("--top-k", type=int, default=0)
    ap.add_argument("--top-p", type=float, default=1.0)
    ap.add_argument("--seed", type=int, default=None)
    ap.add_argument("--eos", type=int, default=None, help="token id that ends a request")
    ap.add_argument("--max-model-len", type=int, default=None, help="default: what the configuration allows, at most 4096")
    ap.add_argument("--max-num-seqs", type=int, default=4)
    ap.add_argument("--block-size", type=int, default=32)
    ap.add_argument("--chunked-prefill", type=int, default=0, metavar="TOKENS",
                    help="token budget of a step: prompts are encoded in portions beside running requests")
    args = ap.parse_args(argv)

    from ._vllm_compat import SamplingParams
    from .engine import MI355XEngine
    from .models import load_config
    config = load_config(args.model)
    max_len = args.max_model_len or min(4096, int(getattr(config, "max_position_embeddings", 4096)))
    override = {"weight_artifacts": False}
    if args.chunked_prefill:
        override.update(is_block_kv_layout=True, chunked_prefill_config={"max_num_seqs": args.max_num_seqs})
    engine = MI355XEngine(config, args.model, dtype=args.dtype, max_model_len=max_len, max_num_seqs=args.max_num_seqs,
                          block_size=args.block_size, enable_prefix_caching=not args.chunked_prefill,
                          enable_chunked_prefill=bool(args.chunked_prefill),
                          max_num_batched_tokens=args.chunked_prefill or None, override_mi355x_config=override)
    prompts = [[int(x) for x in p.split(",") if x.strip()] for p in args.prompt]
    params = SamplingParams(temperature=args.temperature, top_k=args.top_k, top_p=args.top_p, seed=args.seed,
                            max_tokens=args.max_tokens, ignore_eos=args.eos is None)
    for out in engine.generate(prompts, params, eos_token_id=args.eos):
        print(json.dumps({"prompt": out.prompt_token_ids, "tokens": out.token_ids}), flush=True)
    engine.close()
    return 0
