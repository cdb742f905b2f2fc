"""Row ops of decoders with a 32-bit residual stream (HIP kernels in csrc/kernels/residual_norm.hip;
PyTorch reference implementations for CPU processes).

``x`` is always fp32; the second result of ``embed_scale`` / ``residual_rms_norm`` is the same row in the
compute dtype, which the next projection reads (the fp32 tensor itself for an fp32 model).
"""
import torch

from . import native


def embed_scale(table, ids, scale=1.0):
    """x = table[ids] * scale -> (fp32, compute dtype)."""
    if native.use_hip(table):
        return tuple(torch.ops.sxe.embed_scale(table, ids, float(scale)))
    x = table.index_select(0, ids).float() * scale
    return x, x.to(table.dtype)


def residual_rms_norm(x, y, weight, alpha=1.0, eps=1e-6, offset=0.0, index=None, need_x=True):
    """rms(alpha x + y) * (offset + weight) -> (fp32, weight's dtype). ``y`` (the sublayer's output, compute
    dtype) may be None; ``index`` picks rows; ``need_x`` False: only the compute-dtype result is used."""
    if native.use_hip(x):
        return tuple(torch.ops.sxe.residual_rms_norm(x, y, weight, index, float(alpha), float(eps), float(offset),
                                                     bool(need_x)))
    h = alpha * x if y is None else alpha * x + y.float()
    if index is not None:
        h = h.index_select(0, index)
    o = h * torch.rsqrt(h.pow(2).mean(-1, keepdim=True) + eps) * (offset + weight.float())
    return o, o.to(weight.dtype)


def qkv_norm_append(proj, q_norm, k_norm, kc, vc, slots, nq, nkv, dk, dv, eps):
    """``proj`` [T, q | k | v | ...]: RMS norm over the whole q and the whole k projection (plain
    weights), k and v written to ``slots`` of the paged caches [blocks, nkv, bs, D]; returns the
    normalised q [T, nq, D] -- head rows zero-padded to the caches' row length."""
    if native.use_hip(proj):
        return torch.ops.sxe.qkv_norm_append(proj, q_norm, k_norm, kc, vc, slots, int(nq), int(nkv), int(dk), int(dv),
                                             float(eps))
    T, bs = proj.shape[0], kc.shape[2]
    q, k, v = proj[:, :nq * dk + nkv * (dk + dv)].float().split([nq * dk, nkv * dk, nkv * dv], dim=1)
    q = q * torch.rsqrt(q.pow(2).mean(-1, keepdim=True) + eps) * q_norm.float()
    k = k * torch.rsqrt(k.pow(2).mean(-1, keepdim=True) + eps) * k_norm.float()

    def rows(t, n, d, D):
        return torch.nn.functional.pad(t.reshape(T, n, d), (0, D - d)).to(proj.dtype)
    ok = slots >= 0
    s = slots[ok]
    kc[s // bs, :, s % bs] = rows(k, nkv, dk, kc.shape[3])[ok]
    vc[s // bs, :, s % bs] = rows(v, nkv, dv, vc.shape[3])[ok]
    return rows(q, nq, dk, kc.shape[3])


def _rms(x, weight, eps):
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps) * weight.float()


def embed_norm(table, ids, weight, eps, next_weight):
    """x = rms(table[ids]) * weight -> (x fp32, rms(x) * next_weight in the table's dtype)."""
    if native.use_hip(table):
        return tuple(torch.ops.sxe.embed_norm(table, ids, weight, next_weight, float(eps)))
    x = _rms(table.index_select(0, ids).float(), weight, eps)
    return x, _rms(x, next_weight, eps).to(table.dtype)


def sandwich_norm(x, y, post_weight, next_weight, eps, slots=None, add=None, index=None, need_x=True):
    """The sum of a sublayer that has a norm on both sides and the norm in front of the next one, plain
    weights: x' = x + rms(y) * post_weight [+ add] -> (x' fp32, rms(x') * next_weight in y's dtype).

    ``slots`` int32 [T, k]: y's row of token t is the sum of y[slots[t, j]] (expert outputs, one row per
    (token, expert)). ``index`` picks rows; ``need_x`` False: x' itself is not used."""
    if native.use_hip(x):
        return tuple(torch.ops.sxe.sandwich_norm(x, y, post_weight, next_weight, slots, add, index, float(eps), bool(need_x)))
    y = y.float()
    if slots is not None:
        y = y.index_select(0, slots.reshape(-1).long()).view(*slots.shape, -1).sum(1)
    o = x + _rms(y, post_weight, eps)
    if add is not None:
        o = o + add
    if index is not None:
        o = o.index_select(0, index)
    return o, _rms(o, next_weight, eps).to(next_weight.dtype)


def gated_rms_norm(x, weight, gate, eps):
    """rms(x) * weight * sigmoid(gate) over whole rows, plain weight; ``gate`` may be a column slice."""
    if native.use_hip(x):
        return torch.ops.sxe.gated_rms_norm(x, weight, gate, float(eps))
    return (_rms(x.float(), weight, eps) * torch.sigmoid(gate.float())).to(x.dtype)
