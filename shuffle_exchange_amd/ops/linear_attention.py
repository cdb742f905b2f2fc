"""Linear attention with a per-head decay and a carried state (HIP kernels in
csrc/kernels/linear_attn.hip; PyTorch reference form for CPU processes).

Per head S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t. The state [dim, vdim] is fp32 and belongs to the
sequence (RecurrentStates); it counts as zero when a sequence has no earlier tokens.
"""
import math

import torch

from . import native

CHUNK = 256     # tokens of a state chunk of the chunk form
STEP_MAX = 16   # sequences with at most this many new tokens walk token by token
FORMS = {"auto": 0, "step": 1, "chunk": 2}
MIN_LOG2 = -1.0e4  # log2 of a decay of zero


def decay_table(decay, device=None):
    """[2, heads] fp32: the decays and their base-2 logarithms."""
    lg = [math.log2(d) if d > 0 else MIN_LOG2 for d in decay]
    return torch.tensor([list(decay), lg], dtype=torch.float32, device=device)


def decay_attention(proj, state, decay, batch, heads, dim, vdim, act="silu", form="auto"):
    """``proj`` [T, q | k | v | ...] (head by head, before the activation ``act``: "silu" or None);
    ``state`` [slots, heads, dim, vdim] fp32, advanced in place at ``batch.state_slots``; ``decay`` from
    ``decay_table``. Returns o [T, heads * vdim]. ``form``: "step" one token after the other, "chunk" matrix
    products over chunks of tokens (bf16), "auto" by shape. The chunk form leaves the activated k and v in
    ``proj``."""
    if native.use_hip(proj):
        chunk = form == "chunk" or (form == "auto" and chunk_ok(proj, dim, vdim) and max(batch.host_q_len) > STEP_MAX)
        if not chunk:
            return torch.ops.sxe.decay_attention_step(proj, state, decay, batch.q_start, batch.q_len, batch.kv_len,
                                                      batch.state_slots, int(heads), int(dim), int(vdim), act == "silu")
        table = batch.chunks(CHUNK)
        return torch.ops.sxe.decay_attention_chunk(proj, state, decay, batch.q_start, batch.q_len, batch.kv_len,
                                                   batch.state_slots, table, CHUNK, int(heads), int(dim), int(vdim), act == "silu")
    return decay_attention_reference(proj, state, decay, batch, heads, dim, vdim, act)


def chunk_ok(proj, dim, vdim):
    """Shapes of the chunk form: bf16, head sizes up to 128 in multiples of 8."""
    return (proj.dtype == torch.bfloat16 and dim % 8 == 0 and vdim % 8 == 0 and dim <= 128 and vdim <= 128
            and proj.stride(0) % 8 == 0 and proj.data_ptr() % 16 == 0)


def decay_attention_reference(proj, state, decay, batch, heads, dim, vdim, act="silu"):
    qkv = proj[:, :heads * (2 * dim + vdim)].float()
    if act == "silu":
        qkv = torch.nn.functional.silu(qkv)
    qkv = qkv.to(proj.dtype).float()
    q, k, v = (t.unflatten(1, (heads, -1)) for t in qkv.split([heads * dim, heads * dim, heads * vdim], 1))
    out = torch.zeros(proj.shape[0], heads, vdim, dtype=torch.float32, device=proj.device)
    d = decay[0][:, None, None]
    for a, n, kl, slot in zip(*(t.tolist() for t in (batch.q_start, batch.q_len, batch.kv_len, batch.state_slots))):
        S = torch.zeros_like(state[slot]) if kl == n else state[slot].clone()
        for t in range(a, a + n):
            S = d * S + k[t, :, :, None] * v[t, :, None, :]
            out[t] = torch.matmul(q[t, :, None, :], S)[:, 0]
        state[slot] = S
    return out.reshape(proj.shape[0], heads * vdim).to(proj.dtype)
