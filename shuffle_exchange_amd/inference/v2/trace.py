"""Trace replay: feed given token ids through a served model step by step and write logits.

``bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N`` builds the ragged engine
for the checkpoint in DIR (the same ``build_hf_engine`` / ``InferenceEngineV2.put`` that generation
uses) and reads one JSON step a line from standard input:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}], "end": []}

All entries of a step are one ragged batch. The wanted places' logits go to OUT/<step>.f32 (little-endian
fp32 [wanted, vocab], in order; no file when nothing is wanted), then ``done <step>`` is printed;
sequences named in ``end`` are flushed after the step. Nothing is sampled.
"""
import argparse
import json
import math
import os
import sys

import torch

BLOCK = 64


def engine_for_trace(model_dir, dtype, max_tokens, device=None):
    """``max_tokens``: the most tokens that live sequences hold at once."""
    from . import RaggedInferenceEngineConfig, StateManagerConfig, build_hf_engine
    max_tokens = max(1, int(max_tokens))
    seqs = min(max_tokens, 4096)  # every live sequence holds at least one token
    sm = StateManagerConfig(max_tracked_sequences=seqs, max_ragged_batch_size=max_tokens,
                            max_ragged_sequence_count=seqs, max_context=max_tokens)
    # each live sequence may leave one block partly filled; one more block for padded graph rows
    blocks = math.ceil(max_tokens / BLOCK) + min(seqs, 256) + 1
    return build_hf_engine(model_dir, RaggedInferenceEngineConfig(state_manager=sm, kv_block_size=BLOCK,
                                                                  num_kv_blocks=blocks), dtype=dtype, device=device)


def replay(engine, lines, out_dir, done=lambda step: print(f"done {step}", flush=True)):
    uids, free, fresh = {}, [], 0
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = step["entries"]
        for e in entries:
            if e["id"] not in uids:
                if not free:
                    free.append(fresh)
                    fresh += 1
                uids[e["id"]] = free.pop()
        want = [list(e.get("want") or ()) for e in entries]
        if entries:
            logits = engine.put([uids[e["id"]] for e in entries], [torch.tensor(e["tokens"]) for e in entries], want=want)
            if any(want):
                logits.float().cpu().contiguous().numpy().astype("<f4").tofile(
                    os.path.join(out_dir, f"{step['step']}.f32"))
        for name in step.get("end", ()):
            if name in uids:
                uid = uids.pop(name)
                engine.flush(uid)
                free.append(uid)
        done(step["step"])


def main(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a token trace through a served model")
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens held by live requests at any time")
    a = ap.parse_args(argv)
    if not torch.cuda.is_available():
        print("trace_run needs a GPU", file=sys.stderr)
        return 2
    torch.set_float32_matmul_precision("highest")
    from .model_implementations.layered_decoder import ensure_library
    ensure_library(a.model)
    engine = engine_for_trace(a.model, getattr(torch, a.dtype), a.max_tokens)
    replay(engine, sys.stdin, a.out)
    return 0
