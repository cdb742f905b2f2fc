"""Plain fp32 / fp64 implementation of the Tobinex decoder, one function per mechanism.

Slow and independent of the product code: it works on whole sequences with dense [heads, i, j]
score arrays and keeps no cache. Weights are a ``{tensor name: tensor}`` dict with the checkpoint's
names, the configuration is the checkpoint's ``config.json`` dict. Every function takes the dtype of
its inputs as the compute dtype (float64 for reference values).
"""
import math

import torch


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_around_zero(x, w, eps):
    """RMS norm whose stored weight is the deviation from one."""
    return rms(x, eps) * (1.0 + w)


def projection_norm(x, w, eps):
    """RMS norm of a whole projection (all heads together), plain weight."""
    return rms(x, eps) * w


def split_heads(x, n):
    """[T, n * d] -> [n, T, d]."""
    return x.reshape(x.shape[0], n, -1).transpose(0, 1)


def distance_bias(r1, r2, T):
    """[H, T, T]: r1 ln(1 + r2 (i - j)) for j <= i (0 elsewhere: those pairs are masked)."""
    i = torch.arange(T, dtype=r1.dtype)
    d = (i[:, None] - i[None, :]).clamp_min(0)
    return r1[:, None, None] * torch.log(1.0 + r2[:, None, None] * d)


def window_mask(T, size=None, keep_first=0):
    """[T, T] True where position i sees key j: causal, the last ``size`` positions and the first
    ``keep_first`` ones (``size`` None: plain causal)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    m = j <= i
    if size is not None:
        m = m & ((i - j < size) | (j < keep_first))
    return m


def sink_softmax(scores, mask, sink):
    """Softmax over the visible keys with exp(sink_h) added to the denominator."""
    s = scores.masked_fill(~mask, float("-inf"))
    top = torch.maximum(s.amax(-1), sink[:, None])
    e = torch.exp(s - top[..., None])
    return e / (e.sum(-1) + torch.exp(sink[:, None] - top))[..., None]


def talking_heads(weights, talk):
    """weight_h(i, j) <- sum_g talk[h, g] weight_g(i, j)."""
    H = weights.shape[0]
    return (talk @ weights.reshape(H, -1)).reshape(weights.shape)


def attention(h, w, p, m, eps):
    """The attention mixer on one sequence h [T, width]; ``p`` prefix of its tensors, ``m`` its sizes."""
    H, G, T = m["heads"], m["kv_heads"], h.shape[0]
    q = split_heads(projection_norm(h @ w[p + "q"].T, w[p + "q.norm"], eps), H)
    k = split_heads(projection_norm(h @ w[p + "k"].T, w[p + "k.norm"], eps), G)
    v = split_heads(h @ w[p + "v"].T, G)
    kv = torch.arange(H) // (H // G)
    scores = q @ k[kv].transpose(1, 2) * m["scale"] - distance_bias(w[p + "r1"], w[p + "r2"], T)
    mk = m.get("mask") or {}
    probs = sink_softmax(scores, window_mask(T, mk.get("size"), mk.get("keep_first", 0)), w[p + "sink"])
    o = talking_heads(probs, w[p + "talk"]) @ v[kv]
    o = o.transpose(0, 1).reshape(T, -1) * torch.sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def dense_ff(h, w, p):
    g = h @ w[p + "gate"].T
    return (g * torch.sigmoid(g) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def forward(cfg, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one sequence; ``layers_out`` (a list) receives x after every layer."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = norm_around_zero(alpha * x + attention(x, w, p + "mix.", L["mixer"], eps), w[p + "norm1"], eps)
        if L.get("mlp"):
            x = norm_around_zero(alpha * x + dense_ff(x, w, p + "mlp."), w[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x)
    return norm_around_zero(x, w["final.norm"], eps) @ w["embed"].T


def greedy(cfg, weights, prompt, n, dtype=torch.float64):
    ids = [int(t) for t in prompt]
    for _ in range(n):
        ids.append(int(forward(cfg, weights, ids, dtype)[-1].argmax()))
    return ids[len(prompt):]


def random_model(cfg, seed=0, **over):
    """Random bf16-representable weights for ``cfg`` ({name: bf16 tensor}); ``over`` scales a tensor
    kind (its last name component) by a factor."""
    g = torch.Generator().manual_seed(seed)
    D, V = cfg["width"], cfg["vocab"]

    def rnd(*shape, std=1.0, mean=0.0):
        return torch.randn(*shape, generator=g) * std + mean
    w = {"embed": rnd(V, D, std=D ** -0.5), "final.norm": rnd(D, std=0.2)}
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], f"l{i}.mix."
        H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        w[f"l{i}.norm1"] = rnd(D, std=0.2)
        for n, r, c in (("q", H * dk, D), ("k", G * dk, D), ("v", G * dv, D), ("g", H * dv, D), ("o", D, H * dv)):
            w[p + n] = rnd(r, c, std=c ** -0.5)
        w[p + "q.norm"], w[p + "k.norm"] = rnd(H * dk, std=0.2, mean=1.2), rnd(G * dk, std=0.2, mean=1.2)
        w[p + "r1"] = torch.rand(H, generator=g) * 0.8 + 0.05
        w[p + "r2"] = torch.rand(H, generator=g) * 0.5 + 0.02
        w[p + "talk"] = torch.eye(H) * 0.7 + rnd(H, H, std=0.6 / math.sqrt(H))
        w[p + "sink"] = rnd(H, std=0.7)
        if L.get("mlp"):
            F = L["mlp"]["ff"]
            w[f"l{i}.norm2"] = rnd(D, std=0.2)
            w[f"l{i}.mlp.gate"], w[f"l{i}.mlp.up"] = rnd(F, D, std=D ** -0.5), rnd(F, D, std=D ** -0.5)
            w[f"l{i}.mlp.down"] = rnd(D, F, std=F ** -0.5)
    for name in w:
        w[name] = (w[name] * over.get(name.split(".")[-1], 1.0)).to(torch.bfloat16)
    return w
