"""Plain fp32 / fp64 implementation of the Bipotar decoder, one function per mechanism.

Slow and independent of the product code: whole sequences, dense [heads, i, j] score arrays, a
recurrence that walks token by token, no cache. Weights are a ``{tensor name: tensor}`` dict with the
checkpoint's names, the configuration is the checkpoint's ``config.json`` dict. Every function takes the
dtype of its inputs as the compute dtype (float64 for reference values).
"""
import torch


def rms_norm(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def split_heads(x, n):
    """[T, n * d] -> [n, T, d]."""
    return x.reshape(x.shape[0], n, -1).transpose(0, 1)


def rotate_half(x, base, start=0):
    """Rotary positions start, start + 1, ... on the last axis of x [..., T, dims]: component i turns with
    component i + dims/2 by the angle p base^(-2 i / dims)."""
    T, half = x.shape[-2], x.shape[-1] // 2
    f = base ** (-torch.arange(half, dtype=torch.float64) / half)
    a = torch.arange(start, start + T, dtype=torch.float64)[:, None] * f
    c, s = torch.cos(a).to(x.dtype), torch.sin(a).to(x.dtype)
    u, v = x[..., :half], x[..., half:]
    return torch.cat([u * c - v * s, v * c + u * s], -1)


def window_mask(T, size):
    """[T, T] True where i sees j: itself and the size - 1 tokens before it."""
    d = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (d >= 0) & (d < size)


def masked_softmax(scores, mask):
    s = scores.masked_fill(~mask, float("-inf"))
    e = torch.exp(s - s.amax(-1, keepdim=True))
    return e / e.sum(-1, keepdim=True)


def latent_attention(h, w, p, m, eps):
    """Per-head keys [unrotated | shared rotated] and values expanded from the normed latent; h [T, width]."""
    H, T, R = m["heads"], h.shape[0], m["kv_rank"]
    q = split_heads(rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T, H)
    qn, qr = q[..., :m["dim"]], rotate_half(q[..., m["dim"]:], m["rot"]["base"])
    c, kr = (h @ w[p + "dkv"].T).split([R, m["rot_dim"]], -1)
    c, kr = rms_norm(c, w[p + "dkv.norm"], eps), rotate_half(kr, m["rot"]["base"])
    k, v = split_heads(c @ w[p + "uk"].T, H), split_heads(c @ w[p + "uv"].T, H)
    scores = (qn @ k.transpose(1, 2) + qr @ kr.T) * m["scale"]
    o = masked_softmax(scores, window_mask(T, m["mask"]["size"])) @ v
    return o.transpose(0, 1).reshape(T, -1) @ w[p + "o"].T


def decayed_sum(q, k, v, decay):
    """o_t = S_t^T q_t with S_t = decay S_(t-1) + k_t v_t^T, per head: q, k [H, T, d], v [H, T, e]."""
    S = torch.zeros(q.shape[0], q.shape[2], v.shape[2], dtype=q.dtype)
    out = []
    for t in range(q.shape[1]):
        S = decay[:, None, None] * S + k[:, t, :, None] * v[:, t, None, :]
        out.append((q[:, t, None, :] @ S)[:, 0])
    return torch.stack(out, 1)


def lightning(h, w, p, m, eps):
    H = m["heads"]
    q, k, v = (split_heads(silu(h @ w[p + n].T), H) for n in "qkv")
    o = decayed_sum(q, k, v, torch.tensor(m["decay"], dtype=h.dtype))
    o = rms_norm(o.transpose(0, 1).reshape(h.shape[0], -1), w[p + "norm"], eps)
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def dense_ff(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def expert_ff(h, w, p):
    """Squared relu between the two products."""
    return torch.relu(h @ w[p + "up"].T) ** 2 @ w[p + "down"].T


def moe_ff(h, w, p, m):
    """The ``top`` experts with the largest logits, weighted by the softmax over those logits alone."""
    z = h @ w[p + "router"].T
    val, idx = z.topk(m["router"]["top"], dim=-1)
    weight = torch.softmax(val, -1)
    out = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        hit = (weight * (idx == e)).sum(-1, keepdim=True)
        out = out + hit * expert_ff(h, w, f"{p}e{e}.")
    return out


MIXERS = {"latent_attention": latent_attention, "lightning": lightning}


def layer_runs(cfg):
    """[(layer, whether the embedding output is added to x first)] in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop") or {"start": 0, "stop": 0, "times": 1}
    a, b = loop["start"], loop["stop"]
    runs = [(i, False) for i in range(a)]
    for t in range(loop["times"]):
        runs += [(i, t > 0 and i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


def embedding(cfg, w, tokens):
    return rms_norm(w["embed"][torch.as_tensor(tokens)], w["embed.norm"], cfg["norm"]["eps"])


def layer(cfg, w, i, x):
    """x + norm(mixer(norm x)), then x + norm(ff(norm x))."""
    eps, L, p = cfg["norm"]["eps"], cfg["layers"][i], f"l{i}."
    y = MIXERS[L["type"]](rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", L["mixer"], eps)
    x = x + rms_norm(y, w[p + "norm1b"], eps)
    if L.get("mlp"):
        h = rms_norm(x, w[p + "norm2"], eps)
        y = dense_ff(h, w, p + "mlp.") if L["mlp"]["kind"] == "dense" else moe_ff(h, w, p + "mlp.", L["mlp"])
        x = x + rms_norm(y, w[p + "norm2b"], eps)
    return x


def forward(cfg, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one sequence; ``layers_out`` (a list) receives x after every layer run."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    x0 = x = embedding(cfg, w, tokens)
    for i, again in layer_runs(cfg):
        x = layer(cfg, w, i, x + x0 if again else x)
        if layers_out is not None:
            layers_out.append(x)
    return rms_norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["head"].T * cfg["logit_scale"]


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

    def lin(r, c):
        return rnd(r, c, std=c ** -0.5)

    def norm(n):
        return rnd(n, std=0.2, mean=1.0)
    w = {"embed": rnd(V, D, std=0.5), "embed.norm": norm(D), "final.norm": norm(D), "head": lin(V, D)}
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], f"l{i}.mix."
        w[f"l{i}.norm1"], w[f"l{i}.norm1b"] = norm(D), norm(D)
        H = m["heads"]
        if L["type"] == "lightning":
            w[p + "q"], w[p + "k"], w[p + "v"] = lin(H * m["dim"], D), lin(H * m["dim"], D), lin(H * m["vdim"], D)
            w[p + "g"], w[p + "o"], w[p + "norm"] = lin(H * m["vdim"], D), lin(D, H * m["vdim"]), norm(H * m["vdim"])
        else:
            qr, kr = m["q_rank"], m["kv_rank"]
            w[p + "dq"], w[p + "dq.norm"], w[p + "uq"] = lin(qr, D), norm(qr), lin(H * (m["dim"] + m["rot_dim"]), qr)
            w[p + "dkv"], w[p + "dkv.norm"] = lin(kr + m["rot_dim"], D), norm(kr)
            w[p + "uk"], w[p + "uv"], w[p + "o"] = lin(H * m["dim"], kr), lin(H * m["vdim"], kr), lin(D, H * m["vdim"])
        f = L.get("mlp")
        if not f:
            continue
        w[f"l{i}.norm2"], w[f"l{i}.norm2b"] = norm(D), norm(D)
        p = f"l{i}.mlp."
        if f["kind"] == "dense":
            w[p + "gate"], w[p + "up"], w[p + "down"] = lin(f["ff"], D), lin(f["ff"], D), lin(D, f["ff"])
        else:
            w[p + "router"] = lin(f["router"]["experts"], D)
            for e in range(f["router"]["experts"]):
                F = f["expert"]["ff"]
                w[f"{p}e{e}.up"], w[f"{p}e{e}.down"] = lin(F, D), lin(D, F)
    for name in w:
        w[name] = (w[name] * over.get(name.split(".")[-1], 1.0)).to(torch.bfloat16)
    return w
