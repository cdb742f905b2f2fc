"""Paged attention with distance bias, kept-first-keys window, softmax sink, talking heads and output
gate (HIP kernels in csrc/kernels/mix_attn.hip). Every variant is an optional argument, so a design
uses the ones it has.
"""
from dataclasses import dataclass
from typing import Optional

import torch

from . import native
from .paged_attention import choose_splits

FORMS = {"auto": 0, "generic": 1, "token": 2, "tile": 3}
MFMA_ROWS = (64, 128, 256)  # cache row lengths of the matrix-core kernels


def cache_row(d, dtype):
    """Row length of a head of size ``d`` in the paged cache: the next size the matrix-core kernels take
    (rows zero-padded); fp32 models and larger heads keep the size itself."""
    if dtype == torch.bfloat16:
        for D in MFMA_ROWS:
            if d <= D:
                return D
    return d


@dataclass
class MixParams:
    """The fp32 per-head parameters of one layer's attention."""
    r1: Optional[torch.Tensor] = None     # [nq] distance bias r1 ln(1 + r2 (i - j)), subtracted
    r2: Optional[torch.Tensor] = None
    sink: Optional[torch.Tensor] = None   # [nq]
    talk: Optional[torch.Tensor] = None   # [nq, nq]


def mix_attention(q, kc, vc, batch, dk, dv, scale, params, window=None, keep_first=0, gate=None, form="auto"):
    """q [T, nq, D] against the paged k / v caches [blocks, nkv, bs, D] of ``batch`` (RaggedBatch fields)
    -> [T, nq * dv]. ``gate`` [T, nq * dv]: the output is multiplied by its sigmoid. ``form``: which HIP
    kernels ("auto": by shape; "generic" any size, one token per workgroup; "token" scores through
    memory; "tile" 16 tokens x all heads)."""
    if native.use_hip(q):
        splits = _splits(kc, batch, window, keep_first)
        return torch.ops.sxe.mix_attention(q, kc, vc, batch.block_table, batch.q_start, batch.q_len, batch.kv_len,
                                           min(batch.host_q_len), max(batch.host_q_len), int(batch.max_kv_len), splits,
                                           int(dk), int(dv), float(scale), int(window or 0), int(keep_first), params.r1,
                                           params.r2, params.sink, params.talk, gate, FORMS[form])
    return mix_attention_reference(q, kc, vc, batch, dk, dv, scale, params, window, keep_first, gate)


def _splits(kc, batch, window, keep_first):
    return choose_splits(batch.num_seqs, kc.shape[1],
                         batch.max_kv_len if not window else min(batch.max_kv_len, window + keep_first))


def mix_attention_parts(q, kc, vc, batch, dk, dv, scale, params, window=None, keep_first=0, gate=None):
    """Decode (HIP, bf16, one new token per sequence): ``(out, None)`` when the keys fit one split, else
    ``(None, part)`` with part fp32 [splits, T, nq * dv] for ``ops.linear.fused_gatesum_linear``, which
    adds the splits and applies the gate. None where the kernels do not cover the shape."""
    bs, D = kc.shape[2], kc.shape[3]
    if (q.dtype != torch.bfloat16 or D not in MFMA_ROWS or vc.shape[3] != D or bs & (bs - 1) or scale <= 0
            or q.shape[1] > 256 or max(batch.host_q_len) != 1 or q.shape[0] != batch.num_seqs):
        return None
    out, part = torch.ops.sxe.mix_attention_parts(q, kc, vc, batch.block_table, batch.q_start, batch.q_len, batch.kv_len,
                                                  int(batch.max_kv_len), _splits(kc, batch, window, keep_first), int(dk),
                                                  int(dv), float(scale), int(window or 0), int(keep_first), params.r1,
                                                  params.r2, params.sink, params.talk, gate)
    return (out, None) if part.numel() == 0 else (None, part)


def mix_attention_reference(q, kc, vc, batch, dk, dv, scale, params, window=None, keep_first=0, gate=None):
    """PyTorch form over the same paged caches, sequence by sequence, fp32."""
    T, nq, _ = q.shape
    nkv, bs = kc.shape[1], kc.shape[2]
    out = torch.zeros(T, nq, dv, dtype=torch.float32, device=q.device)
    kv_of = torch.arange(nq, device=q.device) // (nq // nkv)
    for s in range(batch.block_table.shape[0]):
        a, n, kl = int(batch.q_start[s]), int(batch.q_len[s]), int(batch.kv_len[s])
        if n == 0:
            continue
        blocks = batch.block_table[s, :(kl + bs - 1) // bs].long()
        k, v = (c[blocks].transpose(0, 1).reshape(nkv, -1, c.shape[-1])[kv_of, :kl, :d].float()
                for c, d in ((kc, dk), (vc, dv)))
        sc = torch.matmul(q[a:a + n, :, :dk].float().transpose(0, 1), k.transpose(1, 2)) * scale
        dist = torch.arange(kl - n, kl, device=q.device)[:, None] - torch.arange(kl, device=q.device)[None, :]
        if params.r1 is not None:
            sc = sc - params.r1[:, None, None] * torch.log(1 + params.r2[:, None, None] * dist.clamp_min(0))
        vis = dist >= 0
        if window:
            vis = vis & ((dist < window) | (torch.arange(kl, device=q.device)[None, :] < keep_first))
        sc = sc.masked_fill(~vis, float("-inf"))
        if params.sink is not None:
            sc = torch.cat([sc, params.sink[:, None, None].expand(nq, n, 1)], -1)
        p = torch.softmax(sc, -1)[..., :kl]
        if params.talk is not None:
            p = torch.matmul(params.talk, p.reshape(nq, -1)).view(nq, n, kl)
        out[a:a + n] = torch.matmul(p, v).transpose(0, 1)
    out = out.reshape(T, nq * dv)
    if gate is not None:
        out = out * torch.sigmoid(gate.float())
    return out.to(q.dtype)
