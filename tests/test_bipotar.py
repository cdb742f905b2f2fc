"""Bipotar through the framework's own entry points (build_hf_engine -> InferenceEngineV2.put / generate)
against the plain implementation in bipotar_oracle.py. Each case runs on the CPU (PyTorch forms of the
ops, fp32) and, marked gpu, on the HIP kernels in fp32 and bf16."""
import json
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import bipotar_oracle as O  # noqa: E402
from shuffle_exchange_amd.inference.v2 import (RaggedInferenceEngineConfig, SchedulingError, StateManagerConfig,  # noqa: E402
                                               build_engine_from_ds_checkpoint, build_hf_engine)
from shuffle_exchange_amd.inference.v2 import trace  # noqa: E402

DEVICES = [pytest.param("cpu", torch.float32, id="cpu"),
           pytest.param("cuda", torch.float32, id="gpu-fp32", marks=pytest.mark.gpu),
           pytest.param("cuda", torch.bfloat16, id="gpu-bf16", marks=pytest.mark.gpu)]


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(E, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": E, "top": top}}


def latent(H, dim, rot, vdim, qr, kr, size, mlp, scale=None, base=10000.0):
    m = {"heads": H, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": qr, "kv_rank": kr, "mask": {"size": size},
         "rot": {"base": base, "dims": rot}, "scale": scale or (dim + rot) ** -0.5}
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def light(H, dim, vdim, mlp, decay=None):
    m = {"heads": H, "dim": dim, "vdim": vdim, "decay": decay or [1 - 2.0 ** -(1 + 7 * i / max(1, H - 1)) for i in range(H)]}
    return {"type": "lightning", "mixer": m, "mlp": mlp}


def config(width, vocab, layers, loop, eps=2e-4, logit_scale=0.7):
    return {"architecture": "Bipotar", "layers": layers, "logit_scale": logit_scale, "norm": {"eps": eps}, "vocab": vocab,
            "width": width, "loop": dict(zip(("start", "stop", "times"), loop))}


CONFIGS = {
    # sizes that are no multiple of anything, one head, a layer without feed-forward, a window of one, all experts chosen,
    # decays of one and (nearly) zero, a loop over the inner layers
    "odd": config(44, 101, [light(3, 9, 5, moe(5, 5, 7), [1.0, 0.3, 1e-9]), latent(3, 7, 6, 11, 13, 10, 24, dense(50)),
                            light(1, 6, 14, None), latent(1, 12, 2, 4, 9, 21, 1, moe(3, 1, 30), base=77.0),
                            latent(2, 5, 4, 6, 20, 8, 40, None)], (1, 3, 3)),
    # matrix-core sizes: padded heads, sorted expert rows, the loop over everything
    "tiles": config(128, 96, [latent(5, 48, 16, 40, 56, 72, 50, moe(4, 2, 128)), light(3, 40, 72, dense(96)),
                              light(4, 128, 128, moe(6, 1, 256))], (0, 3, 2), eps=1e-5),
    # more heads than a tile, a long latent, windows beyond a key tile, a loop that runs once, layers behind the loop
    "wide": config(192, 80, [latent(34, 128, 32, 128, 96, 300, 130, dense(200)), light(2, 64, 24, moe(9, 3, 136)),
                             latent(2, 64, 64, 64, 64, 256, 64, moe(2, 2, 64))], (0, 1, 1)),
    # rows in multiples of 64 throughout, for quantized projections
    "aligned": config(128, 96, [latent(2, 48, 16, 64, 64, 64, 50, dense(192)), light(2, 64, 64, moe(4, 2, 64))], (0, 2, 2)),
    "single": config(64, 64, [latent(4, 16, 8, 16, 24, 32, 20, dense(48))], (0, 0, 1)),
    "state": config(64, 64, [light(4, 16, 16, dense(48), [0.2, 0.9, 0.99, 1.0])], (0, 1, 1)),
}


def sharpened(cfg, seed):
    """Random weights whose attention is far from uniform, so that a wrong key shows."""
    return O.random_model(cfg, seed, uq=2.5)


def checkpoint(tmp_path, name, seed=0, weights=sharpened):
    from safetensors.torch import save_file
    cfg = CONFIGS[name]
    w = weights(cfg, seed)
    d = tmp_path / f"{name}{seed}"
    d.mkdir(exist_ok=True)
    (d / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(d / "model.safetensors"))
    return str(d), cfg, w


def engine(path, device, dtype, blocks=64, block_size=32, **kw):
    return build_hf_engine(path, RaggedInferenceEngineConfig(num_kv_blocks=blocks, kv_block_size=block_size, **kw), dtype=dtype,
                           device=torch.device(device))


def prompt(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def check(got, ref, dtype):
    """fp32: every row within rounding. bf16: nearly every row; a router's close call may send a token to
    another expert, which changes that token's row and, through keys and states, faintly the later ones."""
    d = got.double().cpu() - ref
    d = d - d.mean(-1, keepdim=True)
    err = d.pow(2).mean(-1).sqrt() / ref.std()
    if dtype == torch.float32:
        assert float(err.max()) < 1e-4, f"row {int(err.argmax())}: {float(err.max()):.3e}"
    else:
        assert float(err.median()) < 0.05 and float((err > 0.1).float().mean()) <= 0.1, f"{err.sort(descending=True).values[:8]}"


def run(eng, uid, tokens, cuts):
    """Feed ``tokens`` in portions of the given sizes (the last one repeats); logits of every token."""
    out, at, j = [], 0, 0
    while at < len(tokens):
        n = min(cuts[min(j, len(cuts) - 1)], len(tokens) - at)
        out.append(eng.put([uid], [torch.tensor(tokens[at:at + n])], want=[list(range(n))]).cpu())
        at, j = at + n, j + 1
    return torch.cat(out)


@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("name", ["odd", "tiles", "wide"])
def test_prompt_portions_and_decode(tmp_path, name, device, dtype):
    path, cfg, w = checkpoint(tmp_path, name)
    eng = engine(path, device, dtype)
    toks = prompt(cfg, 150, 1)
    ref = O.forward(cfg, w, toks)
    for cuts in ([150], [1], [2], [3, 5, 2], [70, 1], [31, 1, 2, 64], [32], [17], [100, 33, 1]):
        check(run(eng, 7, toks, cuts), ref, dtype)
        eng.flush(7)
    assert eng.free_blocks >= eng.n_kv_blocks - 1  # one block is the padded graph rows'


@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("name", ["odd", "tiles"])
def test_batches_of_unequal_requests(tmp_path, name, device, dtype):
    path, cfg, w = checkpoint(tmp_path, name, 3)
    eng = engine(path, device, dtype)
    seqs = [prompt(cfg, n, 10 + n) for n in (1, 2, 37, 64, 129, 9)]
    refs = [O.forward(cfg, w, s) for s in seqs]
    # prompts of different lengths in one batch, then a mixed batch (a token here, a portion there), then decode
    heads = [1, 1, 20, 63, 97, 8]
    got = [eng.put(list(range(6)), [torch.tensor(s[:n]) for s, n in zip(seqs, heads)])]
    ref = [torch.stack([r[n - 1] for r, n in zip(refs, heads)])]
    step = {1: 1, 2: 9, 3: 1, 4: 32, 5: 1}
    got.append(eng.put(list(step), [torch.tensor(seqs[u][heads[u]:heads[u] + n]) for u, n in step.items()],
                       want=[[n - 1] if u != 3 else [] for u, n in step.items()]))
    ref.append(torch.stack([refs[u][heads[u] + n - 1] for u, n in step.items() if u != 3]))
    at = {u: heads[u] + n for u, n in step.items()}
    live = [u for u in at if at[u] < len(seqs[u])]
    while live:
        got.append(eng.put(live, [torch.tensor(seqs[u][at[u]:at[u] + 1]) for u in live]))
        ref.append(torch.stack([refs[u][at[u]] for u in live]))
        for u in live:
            at[u] += 1
        live = [u for u in live if at[u] < len(seqs[u])]
    check(torch.cat(got), torch.cat(ref), dtype)


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_freed_blocks_and_state_slots_are_used_again(tmp_path, device, dtype):
    path, cfg, w = checkpoint(tmp_path, "odd", 5)
    eng = engine(path, device, dtype, blocks=12, block_size=16, num_state_slots=2)
    got, ref = [], []
    for r in range(6):  # 12 blocks of 16, 2 + 1 state slots: each round takes what earlier ones filled, in another order
        a, b = prompt(cfg, 40 + 7 * r, 100 + r), prompt(cfg, 75 - 9 * r, 200 + r)
        ra, rb = O.forward(cfg, w, a), O.forward(cfg, w, b)
        got.append(eng.put([0, 1], [torch.tensor(a[:-3]), torch.tensor(b[:-3])]))
        ref.append(torch.stack([ra[-4], rb[-4]]))
        for j in (3, 2, 1):
            got.append(eng.put([1, 0], [torch.tensor([b[-j]]), torch.tensor([a[-j]])]))
            ref.append(torch.stack([rb[-j], ra[-j]]))
        with pytest.raises(SchedulingError):
            eng.put([2], [torch.tensor(prompt(cfg, 16 * 12, 1))])
        with pytest.raises(SchedulingError):  # no state slots left for two more
            eng.put([2, 3], [torch.tensor([1]), torch.tensor([1])])
        eng.flush(r % 2)
        eng.flush(1 - r % 2)
    check(torch.cat(got), torch.cat(ref), dtype)
    assert eng._kv.states.free_slots >= 2


@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("decode", [False, True])
def test_window_at_model_level(tmp_path, device, dtype, decode):
    """One layer: a token just outside the window must not change the logits at all, the ones inside must."""
    path, cfg, _ = checkpoint(tmp_path, "single", 2, O.random_model)
    eng = engine(path, device, dtype)
    W = 20
    cuts = [10_000] if not decode else [40, 1]

    def last(toks, uid):
        y = run(eng, uid, toks, cuts)[-1]
        eng.flush(uid)
        return y
    for n in (21, 64, 65, 70, 97):
        base = prompt(cfg, n, n)
        y0 = last(base, 1)
        for j, seen in ((n - 1 - W, False), (n - W, True), (0, False), (n - 2, True)):
            t = list(base)
            t[j] = (t[j] + 17) % cfg["vocab"]
            diff = float((last(t, 2) - y0).abs().max())
            assert (diff > 1e-4) if seen else diff == 0.0, (n, j, diff)


@pytest.mark.parametrize("device,dtype", DEVICES[:2])
def test_state_reaches_back_to_the_first_token(tmp_path, device, dtype):
    """One recurrent layer with a decay of one: the first token and those around state-chunk edges count."""
    path, cfg, w = checkpoint(tmp_path, "state", 4, O.random_model)
    eng = engine(path, device, dtype)
    n = 600
    base = prompt(cfg, n, 1)
    for j in (0, 255, 256, 511, 512, n - 2):
        t = list(base)
        t[j] = (t[j] + 17) % cfg["vocab"]
        ref = O.forward(cfg, w, t)
        for cuts in ([n], [257, 300, 1]):
            check(run(eng, 0, t, cuts), ref, dtype)
            eng.flush(0)


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_long_decode(tmp_path, device, dtype):
    path, cfg, w = checkpoint(tmp_path, "tiles", 8)
    eng = engine(path, device, dtype)
    toks = prompt(cfg, 330, 4)
    check(run(eng, 0, toks, [3, 1]), O.forward(cfg, w, toks), dtype)


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_first_tokens(tmp_path, device, dtype):
    path, cfg, w = checkpoint(tmp_path, "odd", 9)
    eng = engine(path, device, dtype)
    for n in (1, 2, 3, 6):
        toks = prompt(cfg, n, n)
        for cuts in ([n], [1]):
            check(run(eng, 0, toks, cuts), O.forward(cfg, w, toks), dtype)
            eng.flush(0)


@pytest.mark.gpu
def test_graph_steps_equal_eager_steps(tmp_path):
    """Decode steps replayed from graphs (several buckets, each captured in mid-sequence) advance every state
    exactly once: same logits as an engine without graphs."""
    path, cfg, _ = checkpoint(tmp_path, "tiles", 6)
    a, b = (engine(path, "cuda", torch.bfloat16, decode_graphs=g) for g in (True, False))
    seqs = [prompt(cfg, n, n) for n in (300, 40, 41, 3, 90)]
    for n in (5, 3, 1, 4):
        uids = list(range(n))
        for e in (a, b):
            e.put(uids, [torch.tensor(s[:-30]) if len(s) > 30 else torch.tensor(s[:1]) for s in seqs[:n]])
        for j in range(8):
            t = [torch.tensor([s[-1 - j] if len(s) > 8 else 5]) for s in seqs[:n]]
            torch.testing.assert_close(a.put(uids, t), b.put(uids, t), rtol=2e-2, atol=2e-2)
        for e in (a, b):
            for u in uids:
                e.flush(u)
    assert a._decode_graphs.replays > 0 and not b._decode_graphs


@pytest.mark.parametrize("device,dtype", DEVICES[:2])
def test_greedy_generation(tmp_path, device, dtype):
    path, cfg, w = checkpoint(tmp_path, "odd", 11)
    eng = engine(path, device, dtype)
    prompts = [prompt(cfg, n, n) for n in (5, 1, 33)]
    assert eng.generate(prompts, max_new_tokens=12) == [O.greedy(cfg, w, p, 12) for p in prompts]


@pytest.mark.gpu
def test_greedy_generation_bf16_follows_its_own_logits(tmp_path):
    path, cfg, w = checkpoint(tmp_path, "tiles", 11)
    eng = engine(path, "cuda", torch.bfloat16)
    p = prompt(cfg, 20, 3)
    out = eng.generate([p, p[:7]], max_new_tokens=16)
    for q, o in ((p, out[0]), (p[:7], out[1])):  # the chosen tokens are within rounding of the oracle's best
        ref = O.forward(cfg, w, q + o)[len(q) - 1:-1]
        ok = ref.max(-1).values - ref.gather(1, torch.tensor(o)[:, None])[:, 0] < 0.15 * ref.std()
        assert float(ok.float().mean()) >= 0.9


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_serialized_engine(tmp_path, device, dtype):
    path, cfg, w = checkpoint(tmp_path, "odd", 13)
    eng = engine(path, device, dtype)
    toks = torch.tensor(prompt(cfg, 30, 2))
    y = eng.put([0], [toks]).cpu()
    eng.serialize(str(tmp_path / "saved"))
    if device == "cpu" and torch.cuda.is_available():
        return  # the rebuilt engine takes the process's device
    again = build_engine_from_ds_checkpoint(str(tmp_path / "saved"), RaggedInferenceEngineConfig(num_kv_blocks=8))
    torch.testing.assert_close(again.put([0], [toks]).cpu(), y)


@pytest.mark.gpu
def test_quantized_projections(tmp_path):
    """Dense projections as fp8 weights (experts, latent and router weights stay as they are)."""
    path, cfg, w = checkpoint(tmp_path, "aligned", 25, O.random_model)
    eng = build_hf_engine(path, RaggedInferenceEngineConfig(num_kv_blocks=16), weight_quant="fp8")
    toks = prompt(cfg, 60, 2)
    got, ref = run(eng, 0, toks, [40, 1]).double(), O.forward(cfg, w, toks)
    assert float((got - ref).pow(2).mean(-1).sqrt().median() / ref.std()) < 0.2


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_trace_replay(tmp_path, device, dtype):
    path, cfg, w = checkpoint(tmp_path, "odd", 15)
    a, b = prompt(cfg, 50, 1), prompt(cfg, 20, 2)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:48], "want": [0, 47]}, {"id": "y", "tokens": b[:19], "want": []}]},
             {"step": 1, "entries": [{"id": "x", "tokens": a[48:49], "want": []}, {"id": "y", "tokens": b[19:], "want": [0]}],
              "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": a[49:], "want": [0]}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "x", "tokens": b, "want": [19]}], "end": ["x"]},
             {"step": 4, "entries": [{"id": "z", "tokens": b[:2], "want": []}], "end": ["z"]}]
    eng = trace.engine_for_trace(path, dtype, 80, device=torch.device(device))
    free, done = eng.free_blocks, []
    trace.replay(eng, [json.dumps(s) for s in steps], str(tmp_path), done=done.append)
    assert done == [0, 1, 2, 3, 4] and eng.free_blocks >= free - 1 and not os.path.exists(tmp_path / "4.f32")
    import numpy as np

    def out(n):
        return torch.from_numpy(np.fromfile(tmp_path / f"{n}.f32", dtype="<f4").copy()).view(-1, cfg["vocab"])
    ra, rb = O.forward(cfg, w, a), O.forward(cfg, w, b)
    check(torch.cat([out(n) for n in (0, 1, 2, 3)]), torch.cat([ra[[0, 47]], rb[[19]], ra[[49]], rb[[19]]]), dtype)


def test_layer_by_layer_against_the_oracle(tmp_path):
    """The residual stream after every layer run, looped layers each time."""
    from shuffle_exchange_amd.inference.v2.model_implementations import layered_decoder as M
    path, cfg, w = checkpoint(tmp_path, "odd", 19)
    eng = engine(path, "cpu", torch.float32)
    toks, ref, got = prompt(cfg, 30, 5), [], []
    O.forward(cfg, w, toks, layers_out=ref)
    adds, plain = [], M.sandwich_norm

    def spy(x, y, pw, nw, eps, slots=None, add=None, index=None, need_x=True):
        out = plain(x, y, pw, nw, eps, slots, None, None)[0]
        got.append(out.double())
        adds.append(add is not None)
        return plain(x, y, pw, nw, eps, slots, add, index, need_x)
    M.sandwich_norm = spy
    try:
        eng.put([0], [torch.tensor(toks)])
    finally:
        M.sandwich_norm = plain
    runs, n = [i for i, _ in O.layer_runs(cfg)], -1
    ends = [n := n + (2 if cfg["layers"][i]["mlp"] else 1) for i in runs]
    assert runs == [0, 1, 2, 1, 2, 1, 2, 3, 4] and len(got) == ends[-1] + 1
    for e, r in zip(ends, ref):
        torch.testing.assert_close(got[e], r, rtol=1e-4, atol=1e-4)
    assert [ends.index(i) for i, x in enumerate(adds) if x] == [2, 4]  # ahead of the second and third pass


def test_checkpoint_errors(tmp_path):
    from safetensors.torch import load_file, save_file
    path, cfg, _ = checkpoint(tmp_path, "odd", 17)
    from shuffle_exchange_amd.inference.v2.model_implementations import load_layered_decoder
    with pytest.raises(NotImplementedError):
        load_layered_decoder(path, tp_size=2)
    f = os.path.join(path, "model.safetensors")
    sd = load_file(f)
    save_file({k: v for k, v in sd.items() if k != "l0.mlp.e3.down"}, f)
    with pytest.raises(KeyError, match="l0.mlp.e3.down"):
        engine(path, "cpu", torch.float32)
    save_file({**sd, "l1.mix.uk": sd["l1.mix.uk"][:-1].contiguous()}, f)
    with pytest.raises(ValueError, match="l1.mix.uk"):
        engine(path, "cpu", torch.float32)
    bad = json.loads(json.dumps(cfg))
    bad["loop"]["stop"] = 9
    (tmp_path / "odd17" / "config.json").write_text(json.dumps(bad))
    with pytest.raises(ValueError, match="loop"):
        engine(path, "cpu", torch.float32)


def test_cache_and_state_geometry(tmp_path):
    path, cfg, _ = checkpoint(tmp_path, "odd", 23)
    sm = StateManagerConfig(max_context=64, max_tracked_sequences=5)
    eng = build_hf_engine(path, RaggedInferenceEngineConfig(kv_block_size=16, state_manager=sm), dtype=torch.float32, device="cpu")
    runs = [cfg["layers"][i] for i, _ in O.layer_runs(cfg)]
    rows = sum(L["mixer"]["kv_rank"] + L["mixer"]["rot_dim"] for L in runs if L["type"] == "latent_attention")
    assert eng.n_kv_blocks == 64 * 2**20 // (rows * 16 * 4)
    for r, L in enumerate(runs):
        m = L["mixer"]
        if L["type"] == "lightning":
            assert eng._kv.layer_state(r).shape == (6, m["heads"], m["dim"], m["vdim"])
        else:
            assert eng._kv.layer_kv(r)[0].shape[1:] == (1, 16, m["kv_rank"] + m["rot_dim"])
    only = build_hf_engine(checkpoint(tmp_path, "state", 1)[0], RaggedInferenceEngineConfig(), dtype=torch.float32, device="cpu")
    assert only.put([0], [torch.tensor([1, 2, 3])]).shape == (1, 64)


def test_generate_command_line(tmp_path, capsys):
    from shuffle_exchange_amd.inference.v2 import generate
    path, cfg, w = checkpoint(tmp_path, "odd", 21)
    if torch.cuda.is_available():
        pytest.skip("covered by test_greedy_generation on the GPU")
    assert generate.main(["--model", path, "--prompt", "3,1,4", "--prompt", "1,5", "--max-new-tokens", "4", "--dtype", "float32",
                          "--kv-blocks", "8"]) == 0
    rows = [json.loads(x) for x in capsys.readouterr().out.splitlines() if x.startswith("{")]
    assert [r["generated"] for r in rows] == [O.greedy(cfg, w, p, 4) for p in ([3, 1, 4], [1, 5])]
