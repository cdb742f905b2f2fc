"""Generation from the command line: ``bin/sxe_generate --model DIR --prompt 1,2,3 [--prompt ...]``.

Prompts are token ids (no tokenizer is bundled); all of them run as one continuous batch through
``InferenceEngineV2.generate``. Prints one JSON line per prompt.
"""
import argparse
import json
import sys

import torch


def main(argv=None):
    ap = argparse.ArgumentParser(prog="sxe_generate", description="generate tokens with the ragged engine")
    ap.add_argument("--model", required=True, help="checkpoint folder (config.json and weights)")
    ap.add_argument("--prompt", action="append", required=True, help="comma-separated token ids; repeat for a batch")
    ap.add_argument("--max-new-tokens", type=int, default=32)
    ap.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    ap.add_argument("--top-k", type=int, default=0)
    ap.add_argument("--seed", type=int, default=None)
    ap.add_argument("--eos", type=int, default=None)
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--weight-quant", default=None, help="fp8 | fp6 | fp4 | mxfp8 | int8 ... weight-only quantization")
    ap.add_argument("--kv-blocks", type=int, default=None, help="KV blocks of 64 tokens (default: from free memory)")
    a = ap.parse_args(argv)
    from . import RaggedInferenceEngineConfig, build_hf_engine
    if torch.cuda.is_available():
        from .model_implementations.layered_decoder import ensure_library
        ensure_library(a.model)
    eng = build_hf_engine(a.model, RaggedInferenceEngineConfig(num_kv_blocks=a.kv_blocks), dtype=getattr(torch, a.dtype),
                          weight_quant=a.weight_quant)
    prompts = [[int(x) for x in p.split(",") if x.strip()] for p in a.prompt]
    outs = eng.generate(prompts, max_new_tokens=a.max_new_tokens, temperature=a.temperature, top_k=a.top_k,
                        eos_token_id=a.eos, seed=a.seed)
    for p, o in zip(prompts, outs):
        print(json.dumps({"prompt": p, "generated": o}), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
