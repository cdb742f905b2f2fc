"""Serving throughput of the layered decoders (layered_decoder.py) beside the Llama and Mixtral models at
equal size: prefill and decode tokens/s through ``InferenceEngineV2.put`` with random weights of
real-model layer sizes (``bench.py --serve``).

Every model has the same width, heads, head size, layer count and vocabulary. Tobinex and Llama share the
dense feed-forward width; Tobinex adds its output gate projection, the window (prompts longer than it
attend to fewer keys) and the head mix. Bipotar runs four layers twice -- latent attention + dense, twice
linear attention + experts, latent attention + experts -- and shares Llama's feed-forward width in the dense
layer, Mixtral's experts in the others (without the gate projection). One JSON line per (size, model,
workload).
"""
import json
import time

import torch

# name -> width, heads, kv heads, head size, ff, layers, vocabulary, window, kept first tokens
SIZES = {"8b": (4096, 32, 8, 128, 14336, 8, 32000, 1024, 16),
         "3b": (3072, 24, 8, 128, 8192, 8, 32000, 1024, 16),
         "1b": (2048, 16, 4, 128, 8192, 8, 32000, 512, 4)}
# Bipotar: latent ranks of queries and keys, rotated size, window, experts, chosen, expert ff
LATENT_MOE = {"8b": (1536, 512, 64, 1024, 32, 4, 1792),
              "3b": (1024, 512, 64, 1024, 32, 4, 1536),
              "1b": (768, 256, 64, 512, 16, 2, 1024)}
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


def bipotar_model(size, device):
    from ...ops.linear_attention import decay_table
    from .model_implementations.layered_decoder import (LatentSpec, LayeredSpec, LayerSpec, LinearSpec, LoopSpec, MoESpec,
                                                        RaggedLayeredDecoder)
    D, H, _, d, ff, n, V, _, _ = SIZES[size]
    qr, kr, rot, win, E, top, eff = LATENT_MOE[size]
    latent = LatentSpec(H, d, rot, d, qr, kr, (d + rot) ** -0.5, 10000.0, win)
    light = LinearSpec(H, d, d, [1 - 2.0 ** -(1 + 9 * h / (H - 1)) for h in range(H)])
    moe = MoESpec(E, top, eff)
    spec = LayeredSpec("Bipotar", V, D, 1e-5, norm_offset=0.0, residual="sandwich", loop=LoopSpec(0, 4, n // 4), layers=[
        LayerSpec(latent, ff), LayerSpec(light, moe=moe), LayerSpec(light, moe=moe), LayerSpec(latent, moe=moe)])
    bf = dict(dtype=torch.bfloat16, device=device)

    def w(*shape):
        return torch.randn(*shape, **bf) * shape[-1] ** -0.5

    def one(k):
        return torch.ones(k, **bf)
    W = {"embed": w(V, D), "embed_norm": one(D), "final": one(D), "head": w(V, D), "layers": []}
    for L in spec.layers:
        x = {k: one(D) for k in ("norm1", "norm1b", "norm2", "norm2b")}
        if L.mixer is light:
            x.update(qkvg=w(4 * H * d, D), o_norm=one(H * d), o=w(D, H * d), decay=decay_table(light.decay, device))
        else:
            uk, uv = w(H * d, kr), w(H * d, kr)
            x.update(dqkv=w(qr + kr + rot, D), q_norm=one(qr), kv_norm=one(kr), uq=w(H * (d + rot), qr), uk=uk.view(H, d, kr).transpose(1, 2),
                     uv=uv.view(H, d, kr), ukv=torch.cat([uk, uv]), o=w(D, H * d))
        if L.moe:
            x.update(router=w(E, D), e_up=w(E, eff, D), e_down=w(E, D, eff))
        else:
            x.update(gu=w(2 * ff, D), down=w(D, ff))
        W["layers"].append(x)
    return RaggedLayeredDecoder(spec, W, torch.bfloat16, device)


def mixtral_model(size, device):
    from ...models import MixtralForCausalLM, mixtral_config
    D, H, G, d, _, n, V, _, _ = SIZES[size]
    _, _, _, _, E, top, eff = LATENT_MOE[size]
    cfg = mixtral_config("mixtral-tiny", hidden_size=D, intermediate_size=eff, num_attention_heads=H, num_key_value_heads=G,
                         num_hidden_layers=n, vocab_size=V, max_position_embeddings=16384, num_local_experts=E,
                         num_experts_per_tok=top)
    with torch.device(device):
        return MixtralForCausalLM(cfg).to(torch.bfloat16).eval()


MODELS = {"tobinex": tobinex_model, "bipotar": bipotar_model, "llama": llama_model, "mixtral": mixtral_model}


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
