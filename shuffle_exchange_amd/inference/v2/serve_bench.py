"""Serving throughput of a layered decoder (layered_decoder.py) beside the Llama model at equal size:
prefill and decode tokens/s through ``InferenceEngineV2.put`` with random weights of real-model layer
sizes (``bench.py --serve``).

The Llama model has the same width, heads, head size, feed-forward width, layer count and vocabulary; the
layered design adds its output gate projection, the window (prompts longer than it attend to fewer keys)
and the head mix. One JSON line per (size, model, workload).
"""
import json
import time

import torch

# name -> width, heads, kv heads, head size, ff, layers, vocabulary, window, kept first tokens
SIZES = {"8b": (4096, 32, 8, 128, 14336, 8, 32000, 1024, 16),
         "3b": (3072, 24, 8, 128, 8192, 8, 32000, 1024, 16),
         "1b": (2048, 16, 4, 128, 8192, 8, 32000, 512, 4)}
PREFILL = ((1, 2048), (4, 2048), (1, 8192))      # (sequences, tokens each)
DECODE = ((1, 2048), (4, 2048), (32, 2048), (128, 2048))  # (sequences, context)


def tobinex_model(size, device):
    from .model_implementations.layered_decoder import (AttentionSpec, LayeredSpec, LayerSpec, RaggedLayeredDecoder)
    D, H, G, d, ff, n, V, win, keep = SIZES[size]
    spec = LayeredSpec("Tobinex", V, D, 1e-5, (2 * n) ** 0.25, D ** 0.5, 1.0,
                       [LayerSpec(AttentionSpec(H, G, d, d, d ** -0.5, win, keep), ff) for _ in range(n)])
    bf = dict(dtype=torch.bfloat16, device=device)

    def w(*shape):
        return torch.randn(*shape, **bf) * shape[-1] ** -0.5
    W = {"embed": w(V, D), "final": torch.zeros(D, **bf), "layers": []}
    for _ in range(n):
        W["layers"].append({"norm1": torch.zeros(D, **bf), "norm2": torch.zeros(D, **bf), "qkvg": w((2 * H + 2 * G) * d, D),
                            "q_norm": torch.ones(H * d, **bf), "k_norm": torch.ones(G * d, **bf), "o": w(D, H * d),
                            "r1": torch.rand(H, device=device), "r2": torch.rand(H, device=device) * 0.5,
                            "sink": torch.randn(H, device=device), "gu": w(2 * ff, D), "down": w(D, ff),
                            "talk": torch.eye(H, device=device) + torch.randn(H, H, device=device) * 0.5 * H ** -0.5})
    return RaggedLayeredDecoder(spec, W, torch.bfloat16, device)


def llama_model(size, device):
    from ...models import LlamaForCausalLM, llama_config
    D, H, G, d, ff, n, V, _, _ = SIZES[size]
    cfg = llama_config("llama-tiny", hidden_size=D, intermediate_size=ff, num_attention_heads=H, num_key_value_heads=G,
                       num_hidden_layers=n, vocab_size=V, max_position_embeddings=16384)
    with torch.device(device):
        return LlamaForCausalLM(cfg).to(torch.bfloat16).eval()


MODELS = {"tobinex": tobinex_model, "llama": llama_model}


def run(sizes=None, models=None, steps=16, warmup=4, emit=lambda row: print(json.dumps(row), flush=True), prefill=PREFILL,
        decode=DECODE):
    from . import InferenceEngineV2, RaggedInferenceEngineConfig, StateManagerConfig
    device = torch.device("cuda", torch.cuda.current_device())
    rows = []

    def timed(f, n):
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        for _ in range(n):
            f()
        torch.cuda.synchronize()
        return (time.perf_counter() - t0) / n * 1e3
    for size in sizes or SIZES:
        for name in models or MODELS:
            torch.manual_seed(0)
            eng = InferenceEngineV2(MODELS[name](size, device), RaggedInferenceEngineConfig(
                kv_block_size=64, num_kv_blocks=128 * 40, state_manager=StateManagerConfig(max_ragged_batch_size=16384)))
            V = SIZES[size][6]
            g = torch.Generator().manual_seed(1)

            def row(kind, n, length, ms, toks):
                rows.append({"bench": "serve", "size": size, "model": name, "workload": kind, "sequences": n, "tokens": length,
                             "ms": round(ms, 3), "tokens_per_s": round(toks / ms * 1e3, 1), "dtype": "bf16",
                             "data": "synthetic, random weights", "layers": SIZES[size][5]})
                emit(rows[-1])
            for n, length in prefill:
                toks = [torch.randint(0, V, (length,), generator=g) for _ in range(n)]

                def once():
                    eng.put(list(range(n)), toks)
                    for u in range(n):
                        eng.flush(u)
                for _ in range(2):
                    once()
                row("prefill", n, length, timed(once, max(2, steps // 2)), n * length)
            for n, length in decode:
                for u in range(n):
                    eng.put([u], [torch.randint(0, V, (length,), generator=g)])
                nxt = [torch.tensor([1])] * n
                for _ in range(warmup):
                    eng.put(list(range(n)), nxt)
                row("decode", n, length, timed(lambda: eng.put(list(range(n)), nxt), steps), n)
                for u in range(n):
                    eng.flush(u)
            del eng
            torch.cuda.empty_cache()
    return rows
