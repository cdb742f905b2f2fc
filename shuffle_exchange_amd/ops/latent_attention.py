"""Attention over a cached low-rank latent (HIP kernels in csrc/kernels/latent_attn.hip; PyTorch reference
forms for CPU processes).

A token's cache row is [latent c | rotated key part shared by all heads], one row for all heads. Per head
the unrotated key is W_uk c and the value W_uv c, so

  score = (q_n . W_uk c + rot(q_r) . k_r) scale = ((W_uk^T q_n) . c + rot(q_r) . k_r) scale
  out   = sum_j p_j W_uv c_j = W_uv (sum_j p_j c_j)

The left forms expand keys and values (prompts: fewer operations per key), the right ones stay in the
latent (decode: the cache row is read once for all heads).
"""
import torch

from . import native

TILE_MIN = 32          # sequences with at least this many new tokens take the expanded form
PAD_RANK, PAD_ROT = 128, 64  # bf16 cache rows: the parts' lengths are padded to multiples of these


def latent_row(rank, rot, dtype):
    """(latent length, rotated length) of a cache row; bf16 rows are zero-padded for the matrix cores."""
    if dtype == torch.bfloat16:
        return -(-rank // PAD_RANK) * PAD_RANK, -(-rot // PAD_ROT) * PAD_ROT
    return rank, rot


def rotation_table(positions, dims, base):
    """fp32 [T, dims / 2, 2]: cos and sin of p base^(-2 i / dims). Angles are formed in fp64 and reduced before
    they are rounded."""
    if native.use_hip(positions):
        return torch.ops.sxe.rotation_table(positions, int(dims), float(base))
    f = float(base) ** (-torch.arange(dims // 2, dtype=torch.float64) * 2 / dims)
    a = positions.double()[:, None] * f
    return torch.stack([torch.cos(a), torch.sin(a)], -1).float()


def rotate(x, rot):
    """Rotate-half pairs (i, i + dims / 2) of the last axis of x [T, n, dims] (fp32) by ``rotation_table``."""
    c, s = rot[:, None, :, 0], rot[:, None, :, 1]
    u, v = x.chunk(2, -1)
    return torch.cat([u * c - v * s, v * c + u * s], -1)


def latent_append(proj, q_norm, kv_norm, cache, slots, rot, q_rank, rank, rot_dim, eps):
    """``proj`` [T, query latent | latent | key part]: both latents RMS-normed (plain weights), the key part
    rotated, latent and key part written to ``slots`` of the paged ``cache`` [blocks, 1, bs, row];
    returns the normed query latent [T, q_rank]."""
    R, _ = latent_row(rank, rot_dim, proj.dtype)
    if native.use_hip(proj):
        return torch.ops.sxe.latent_append(proj, q_norm, kv_norm, cache, slots, rot, int(q_rank), int(rank), int(R),
                                           int(rot_dim), float(eps))
    cq, c, kr = proj.float().split([q_rank, rank, rot_dim], 1)

    def norm(x, w):
        return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps) * w.float()
    row = torch.zeros(proj.shape[0], cache.shape[3], dtype=cache.dtype, device=cache.device)
    row[:, :rank] = norm(c, kv_norm).to(cache.dtype)
    row[:, R:R + rot_dim] = rotate(kr[:, None], rot)[:, 0].to(cache.dtype)
    ok, bs = slots >= 0, cache.shape[2]
    cache[slots[ok] // bs, 0, slots[ok] % bs] = row[ok]
    return norm(cq, q_norm).to(proj.dtype)


def latent_attention(q, uk, uv, ukv, cache, batch, rot, heads, dim, rot_dim, vdim, rank, scale, window=None, form="auto"):
    """``q`` [T, heads * (dim + rot_dim)] (per head [unrotated | to be rotated]) against the paged latent
    ``cache``; ``uk`` [heads, rank, dim] and ``uv`` [heads, vdim, rank] (the product's inner dimension last), ``ukv``
    [heads * (dim + vdim), rank] the same weights stacked key rows first (None: the expanded form is not used). Returns [T, heads * vdim].

    ``form``: "token" one token's heads against the latents, "tile" keys and values expanded for tiles of
    tokens, "generic" any size and dtype, "auto" by shape (sequences of a batch may take different forms)."""
    if not native.use_hip(q):
        return latent_attention_reference(q, uk, uv, cache, batch, rot, heads, dim, rot_dim, vdim, rank, scale, window)
    R, _ = latent_row(rank, rot_dim, q.dtype)
    if form == "auto":
        tile = ukv is not None and tile_ok(q, dim, rot_dim, vdim) and max(batch.host_q_len) >= TILE_MIN
        least = TILE_MIN if tile and min(batch.host_q_len) < TILE_MIN else 1
        token = token_ok(q, dim, rot_dim, rank, R, scale)
    else:
        tile, least, token = form == "tile", 1, form == "token"
    out = torch.empty(q.shape[0], heads * vdim, dtype=q.dtype, device=q.device)
    w = int(window or 0)
    lens = (batch.q_start, batch.q_len, batch.kv_len)
    if tile:
        slots, first = batch.key_rows(window, least)
        lat = cache.view(-1, cache.shape[3]).index_select(0, slots)
        kv = torch.nn.functional.linear(lat[:, :rank], ukv)
        torch.ops.sxe.latent_attention_tile(q, kv, lat, rot, batch.chunks(TILE_TOKENS, least), TILE_TOKENS, first, *lens, out,
                                            int(heads), int(dim), int(rot_dim), int(vdim), int(R), float(scale), w)
        if least == 1:
            return out
    rows = batch.token_rows(TILE_MIN if tile else None)  # tokens of the other sequences
    if token:
        keys = int(batch.max_kv_len) if not w else min(int(batch.max_kv_len), w)
        wgs = max(1, rows.shape[0] * -(-heads // TOKEN_HEADS))
        splits = max(1, min(-(-keys // TOKEN_KEYS), TOKEN_WGS // wgs))
        torch.ops.sxe.latent_attention_token(q, uk, uv, cache, rot, rows, batch.block_table, *lens, out, splits, int(rot_dim),
                                             int(R), float(scale), w)
    else:
        torch.ops.sxe.latent_attention_generic(q, uk, uv, cache, rot, rows, batch.block_table, *lens, out, int(rot_dim), int(R),
                                               float(scale), w)
    return out


TOKEN_HEADS, TOKEN_KEYS, TOKEN_WGS = 32, 64, 256  # token form: heads and keys of a tile; workgroups to aim for with key splits
TILE_TOKENS = 256  # query tokens of a workgroup of the expanded form


def tile_ok(q, dim, rot_dim, vdim):
    return (q.dtype == torch.bfloat16 and dim <= 128 and rot_dim <= 64 and vdim <= 128 and dim % 8 == 0 and rot_dim % 8 == 0
            and vdim % 8 == 0 and q.data_ptr() % 16 == 0)


def token_ok(q, dim, rot_dim, rank, R, scale):
    return (q.dtype == torch.bfloat16 and R <= 512 and rot_dim <= 64 and scale > 0 and dim % 8 == 0 and rank % 8 == 0
            and rot_dim % 8 == 0 and q.data_ptr() % 16 == 0)


def latent_attention_reference(q, uk, uv, cache, batch, rot, heads, dim, rot_dim, vdim, rank, scale, window=None):
    """PyTorch form over the same paged cache, sequence by sequence, fp32."""
    T, bs = q.shape[0], cache.shape[2]
    R, _ = latent_row(rank, rot_dim, q.dtype)
    qn, qr = q.float().view(T, heads, dim + rot_dim).split([dim, rot_dim], -1)
    qr = rotate(qr, rot)
    out = torch.zeros(T, heads, vdim, dtype=torch.float32, device=q.device)
    for s in range(batch.block_table.shape[0]):
        a, n, kl = int(batch.q_start[s]), int(batch.q_len[s]), int(batch.kv_len[s])
        if n == 0:
            continue
        rows = cache[batch.block_table[s, :(kl + bs - 1) // bs].long(), 0].reshape(-1, cache.shape[3])[:kl].float()
        c, kr = rows[:, :rank], rows[:, R:R + rot_dim]
        k, v = torch.matmul(c, uk.float()), torch.matmul(c, uv.float().transpose(1, 2))
        sc = torch.matmul(qn[a:a + n].transpose(0, 1), k.transpose(1, 2))
        sc = (sc + torch.matmul(qr[a:a + n].transpose(0, 1), kr.t())) * scale
        dist = torch.arange(kl - n, kl, device=q.device)[:, None] - torch.arange(kl, device=q.device)[None, :]
        vis = dist >= 0
        if window:
            vis = vis & (dist < window)
        out[a:a + n] = torch.matmul(torch.softmax(sc.masked_fill(~vis, float("-inf")), -1), v).transpose(0, 1)
    return out.reshape(T, heads * vdim).to(q.dtype)
