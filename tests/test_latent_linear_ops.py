"""ops/latent_attention.py, ops/linear_attention.py, the routed experts of ops/moe.py and the sandwich norms of
ops/residual_norm.py against the plain functions of bipotar_oracle.py: the PyTorch forms on the CPU, every
HIP form on the GPU."""
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import bipotar_oracle as O  # noqa: E402
from shuffle_exchange_amd.inference.v2.ragged.ragged import DSSequenceDescriptor, RaggedBatch  # noqa: E402
from shuffle_exchange_amd.ops import latent_attention as LA  # noqa: E402
from shuffle_exchange_amd.ops import linear_attention as LN  # noqa: E402
from shuffle_exchange_amd.ops import moe as ME  # noqa: E402
from shuffle_exchange_amd.ops import residual_norm as RN  # noqa: E402

gpu = pytest.mark.gpu
DEVICES = [pytest.param("cpu", torch.float32, id="cpu"), pytest.param("cuda", torch.float32, id="gpu-fp32", marks=gpu),
           pytest.param("cuda", torch.bfloat16, id="gpu-bf16", marks=gpu)]


def rounded(t, dtype):
    return t.to(dtype).double()


def close(got, ref, tol, what=""):
    """Largest error of a row relative to the rows' root mean square."""
    d = (got.double().cpu() - ref).reshape(ref.shape[0], -1)
    e = d.pow(2).mean(-1).sqrt() / ref.pow(2).mean().sqrt()
    assert torch.isfinite(e).all() and float(e.max()) < tol, f"{what}: row {int(e.argmax())}: {float(e.max()):.3e}"


def make_batch(lens, bs, device, seed=0, extra=3):
    """RaggedBatch of (history, new tokens) sequences over shuffled blocks and state slots; block count."""
    g = torch.Generator().manual_seed(seed)
    nb = [-(-(a + n) // bs) for a, n in lens]
    perm, at, seqs = torch.randperm(sum(nb) + extra, generator=g).tolist(), 0, []
    slot = torch.randperm(len(lens) + 2, generator=g).tolist()
    for i, (a, n) in enumerate(lens):
        seqs.append(DSSequenceDescriptor(i, 1 << 20, slot[i], a, 0, perm[at:at + nb[i]]))
        at += nb[i]
    toks = [torch.zeros(n, dtype=torch.int64) for _, n in lens]
    return RaggedBatch(seqs, toks, bs, torch.device(device)), sum(nb) + extra, len(lens) + 2


# ---------------------------------------------------------------------------------------- linear attention
def linear_case(lens, H, d, e, decay, dtype, device, form, seed=0, spike=None):
    g = torch.Generator().manual_seed(seed)
    batch, _, nslots = make_batch(lens, 16, device, seed)
    T = sum(n for _, n in lens)
    proj = torch.randn(T, H * (2 * d + 2 * e) + 8, generator=g)
    if spike is not None:  # one token's key and value stand out
        proj[spike, H * d:H * (2 * d + e)] = 4.0
    proj = proj.to(dtype)
    state = torch.randn(nslots, H, d, e, generator=g) * 2
    state0 = state.clone()
    for s, (a, n) in enumerate(lens):
        if a == 0:
            state[int(batch.state_slots[s])] = float("nan")  # whatever the slot's last owner left
    st = state.to(device)
    out = LN.decay_attention(proj.to(device), st, LN.decay_table(decay, device), batch, H, d, e, form=form)
    act = rounded(O.silu(proj.double()), dtype)
    refs, row = [], 0
    dec = torch.tensor(decay, dtype=torch.float64)
    for s, (a, n) in enumerate(lens):
        q, k, v = act[row:row + n, :H * (2 * d + e)].split([H * d, H * d, H * e], 1)
        q, k, v = (O.split_heads(x, H) for x in (q, k, v))
        S0 = state0[int(batch.state_slots[s])].double() if a else torch.zeros(H, d, e, dtype=torch.float64)
        o = O.decayed_sum(q, k, v, dec)
        p = dec[:, None] ** torch.arange(1, n + 1)
        o = o + p[..., None] * (q @ S0)
        refs.append(o.transpose(0, 1).reshape(n, H * e))
        S1 = dec[:, None, None] ** n * S0 + torch.einsum("htd,hte->hde", k * (dec[:, None] ** torch.arange(n - 1, -1, -1))[..., None], v)
        close(st[int(batch.state_slots[s])], S1, 2e-4 if dtype == torch.bfloat16 else 2e-5, f"state {s}")
        row += n
    # rows differ in size by orders (a token soon after a spike): compare row by row
    ref = torch.cat(refs)
    err = (out.double().cpu() - ref).pow(2).mean(-1).sqrt() / ref.pow(2).mean(-1).sqrt()
    assert float(err.max()) < (2e-2 if dtype == torch.bfloat16 else 2e-5), f"row {int(err.argmax())}: {float(err.max()):.3e}"


DECAY = [0.2, 0.9, 0.99, 1.0]


@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("d,e", [(16, 8), (9, 5), (64, 96), (130, 36)])
def test_linear_attention_step_form(d, e, device, dtype):
    linear_case([(0, 1), (5, 1), (300, 1), (0, 40), (7, 16), (3, 2)], 4, d, e, DECAY, dtype, device, "step")


@gpu
@pytest.mark.parametrize("d,e", [(16, 8), (64, 64), (64, 128), (128, 64), (128, 128), (72, 40)])
def test_linear_attention_chunk_form(d, e):
    lens = [(0, 700), (9, 255), (0, 1), (4, 256), (0, 257), (100, 64), (3, 1), (0, 129)]
    linear_case(lens, 4, d, e, DECAY, torch.bfloat16, "cuda", "chunk")


@gpu
@pytest.mark.parametrize("spike", [0, 31, 63, 64, 127, 128, 255, 256, 510])
def test_linear_attention_far_token(spike):
    linear_case([(0, 512)], 2, 64, 64, [0.97, 1.0], torch.bfloat16, "cuda", "chunk", spike=spike)


def test_decay_table():
    t = LN.decay_table([1.0, 0.5, 0.0])
    assert t.tolist() == [[1.0, 0.5, 0.0], [0.0, -1.0, LN.MIN_LOG2]]


# --------------------------------------------------------------------------------------- latent attention
def latent_case(lens, H, dim, rd, vdim, R, window, dtype, device, form, bs=32, seed=0, needle=None, scale=None):
    """Cache rows written through latent_append, then attention. ``needle`` (sequence, key, weight): that key's
    latent and rotated part get a large component along every head's query."""
    g = torch.Generator().manual_seed(seed)
    batch, nblocks, _ = make_batch(lens, bs, device, seed)
    Rp, rp = LA.latent_row(R, rd, dtype)
    cache = torch.randn(nblocks, 1, bs, Rp + rp, generator=g)
    cache[..., R:Rp] = 0
    cache[..., Rp + rd:] = 0
    cache = cache.to(dtype)
    scale = scale or (dim + rd) ** -0.5
    base = 500.0
    uk = rounded(torch.randn(H * dim, R, generator=g) * R ** -0.5, dtype)
    uv = rounded(torch.randn(H * vdim, R, generator=g) * R ** -0.5, dtype)
    qs, refs = [], []
    for s, (a, n) in enumerate(lens):
        c = rounded(torch.randn(a + n, R, generator=g), dtype)
        kr = rounded(torch.randn(a + n, rd, generator=g), dtype)  # rotated already
        q = rounded(torch.randn(n, H, dim + rd, generator=g), dtype)
        if needle is not None and needle[0] == s:
            qa = torch.einsum("thd,hdr->r", q[..., :dim], uk.view(H, dim, R))
            c[needle[1]] = rounded(c[needle[1]] + needle[2] * qa / qa.norm() * R ** 0.5, dtype)
        qs.append(q)
        for j in range(a + n):
            blk = int(batch.block_table[s, j // bs])
            cache[blk, 0, j % bs, :R] = c[j].to(dtype)
            cache[blk, 0, j % bs, Rp:Rp + rd] = kr[j].to(dtype)
        qn, qr = q.transpose(0, 1)[..., :dim], O.rotate_half(q.transpose(0, 1)[..., dim:], base, a)
        k, v = O.split_heads(c @ uk.T, H), O.split_heads(c @ uv.T, H)
        sc = (qn @ k.transpose(1, 2) + qr @ kr.T) * scale
        m = O.window_mask(a + n, window)[a:] if window else O.window_mask(a + n, a + n + 1)[a:]
        refs.append((O.masked_softmax(sc, m) @ v).transpose(0, 1).reshape(n, -1))
    q = torch.cat(qs).reshape(-1, H * (dim + rd)).to(dtype).to(device)
    rot = LA.rotation_table(batch.positions, rd, base)
    ukd, uvd = uk.to(dtype).to(device), uv.to(dtype).to(device)
    args = (ukd.view(H, dim, R).transpose(1, 2).contiguous(), uvd.view(H, vdim, R), torch.cat([ukd, uvd]), cache.to(device))
    kw = {} if form is None else {"form": form}
    out = LA.latent_attention(q, *args, batch, rot, H, dim, rd, vdim, R, scale, window, **kw)
    close(out, torch.cat(refs), 2e-2 if dtype == torch.bfloat16 else 2e-5, form)


LENS = [(0, 1), (0, 2), (100, 1), (31, 1), (63, 2), (200, 7), (32, 1)]


@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("window", [None, 1, 33, 64])
def test_latent_attention_generic_form(window, device, dtype):
    latent_case(LENS, 3, 10, 6, 7, 21, window, dtype, device, "generic")


@gpu
@pytest.mark.parametrize("H,dim,rd,vdim,R", [(5, 48, 32, 40, 112), (34, 128, 64, 128, 512), (3, 24, 8, 12, 248), (16, 32, 32, 36, 320),
                                             (1, 8, 8, 5, 8), (2, 200, 48, 20, 136)])
@pytest.mark.parametrize("window", [None, 1, 33, 64, 128])
def test_latent_attention_token_form(window, H, dim, rd, vdim, R):
    latent_case(LENS, H, dim, rd, vdim, R, window, torch.bfloat16, "cuda", "token")


@gpu
def test_latent_attention_token_form_large_batch_and_key_splits():
    latent_case([(j * 7, 1) for j in range(70)], 5, 32, 16, 24, 64, 200, torch.bfloat16, "cuda", "token")
    latent_case([(1500, 1)], 5, 32, 16, 24, 64, None, torch.bfloat16, "cuda", "token")


@gpu
@pytest.mark.parametrize("H,dim,rd,vdim", [(3, 56, 48, 64), (2, 128, 64, 128), (4, 40, 8, 72), (2, 96, 32, 24)])
@pytest.mark.parametrize("window", [None, 1, 50, 64, 130])
def test_latent_attention_tile_form(window, H, dim, rd, vdim):
    latent_case([(0, 300), (77, 128), (500, 1), (0, 2), (130, 129)], H, dim, rd, vdim, 72, window, torch.bfloat16, "cuda", "tile")


@gpu
def test_latent_attention_forms_mixed_in_a_batch():
    latent_case([(0, 90), (300, 1), (40, 2), (64, 33), (9, 31)], 3, 80, 48, 56, 104, 50, torch.bfloat16, "cuda", None)


@gpu
@pytest.mark.parametrize("form", ["generic", "token", "tile"])
@pytest.mark.parametrize("key", [35, 36, 0, 63, 64, 99])
def test_latent_attention_needle_at_the_window_edge(form, key):
    """One query at position 99 with a window of 64 (sees 36 ..): a key that dominates if it is visible."""
    latent_case([(99, 1), (0, 70)], 2, 32, 16, 32, 64, 64, torch.bfloat16, "cuda", form, needle=(0, key, 6.0))


@pytest.mark.parametrize("device", ["cpu", pytest.param("cuda", marks=gpu)])
def test_rotation_table_far_positions(device):
    p = torch.tensor([0, 1, 1000, 123_457, 10_000_019], device=device)
    t = LA.rotation_table(p, 10, 77.0).double().cpu()
    a = p.cpu().double()[:, None] * 77.0 ** (-torch.arange(5, dtype=torch.float64) / 5)
    torch.testing.assert_close(t, torch.stack([a.cos(), a.sin()], -1), rtol=0, atol=1e-6)


@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("qr,R,rd", [(24, 16, 8), (13, 21, 6), (1536, 512, 64)])
def test_latent_append(qr, R, rd, device, dtype):
    batch, nblocks, _ = make_batch([(0, 3), (37, 2), (15, 1)], 16, device)
    Rp, rp = LA.latent_row(R, rd, dtype)
    g = torch.Generator().manual_seed(1)
    proj, qw, kw = (torch.randn(*s, generator=g).to(dtype) for s in ((6, qr + R + rd), (qr,), (R,)))
    cache = torch.zeros(nblocks, 1, 16, Rp + rp, dtype=dtype, device=device)
    rot = LA.rotation_table(batch.positions, rd, 100.0)
    cq = LA.latent_append(proj.to(device), qw.to(device), kw.to(device), cache, batch.slots, rot, qr, R, rd, 1e-5)
    tol = 1e-2 if dtype == torch.bfloat16 else 1e-5
    p = proj.double()
    close(cq, O.rms_norm(p[:, :qr], qw.double(), 1e-5), tol)
    rows = cache.view(-1, Rp + rp)[batch.slots].cpu()
    close(rows[:, :R], O.rms_norm(p[:, qr:qr + R], kw.double(), 1e-5), tol)
    for i, pos in enumerate(batch.positions.tolist()):
        close(rows[i:i + 1, Rp:Rp + rd], O.rotate_half(p[i:i + 1, qr + R:], 100.0, pos), tol)
    written = torch.zeros(cache.shape[0] * 16, dtype=torch.bool)
    written[batch.slots.cpu()] = True
    assert not cache.cpu().view(-1, Rp + rp)[~written].any() and not rows[:, R:Rp].any() and not rows[:, Rp + rd:].any()


# ----------------------------------------------------------------------------------------------- experts
@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("T,E,k,D,F", [(1, 4, 2, 32, 24), (7, 5, 5, 44, 30), (130, 9, 1, 64, 40), (70, 3, 2, 128, 128),
                                       (900, 2, 1, 256, 256), (400, 70, 3, 128, 128), (3, 100, 6, 2048, 16)])
def test_routed_experts(T, E, k, D, F, device, dtype):
    g = torch.Generator().manual_seed(T)
    h = torch.randn(T, D, generator=g).to(dtype)
    w = {"router": torch.randn(E, D, generator=g) * D ** -0.5}
    for e in range(E):
        w[f"e{e}.up"], w[f"e{e}.down"] = torch.randn(F, D, generator=g) * D ** -0.5, torch.randn(D, F, generator=g) * F ** -0.5
    w = {n: t.to(dtype) for n, t in w.items()}
    ref = O.moe_ff(h.double(), {n: t.double() for n, t in w.items()}, "", {"router": {"experts": E, "top": k}})
    up, down = (torch.stack([w[f"e{e}.{n}"] for e in range(E)]).to(device) for n in ("up", "down"))
    hd = h.to(device)
    routing = ME.route_topk(hd, w["router"].to(device), k)
    idx, wt = routing[:2]
    z = h.double() @ w["router"].double().T
    val, ri = z.topk(k, dim=-1)
    torch.testing.assert_close(wt.double().cpu(), torch.softmax(val, -1), rtol=2e-5, atol=1e-6)
    assert torch.equal(idx.cpu().long(), ri)  # the fp32 order of random logits
    y, slots = ME.expert_mlp(hd, routing, up, down)
    assert sorted(slots.cpu().reshape(-1).tolist()) == list(range(T * k))
    got = y.cpu().double()[slots.cpu().long().reshape(-1)].view(T, k, D).sum(1)
    close(got, ref, 2e-2 if dtype == torch.bfloat16 else 2e-5)


@gpu
def test_route_topk_prefers_the_lower_index_and_survives_nan():
    h = torch.zeros(3, 32, dtype=torch.bfloat16, device="cuda")
    h[2] = float("nan")
    idx, wt = ME.route_topk(h, torch.randn(12, 32, device="cuda").to(torch.bfloat16), 4)[:2]
    assert idx[:2].tolist() == [[0, 1, 2, 3]] * 2 and bool((wt[:2] == 0.25).all())
    assert bool(((idx >= 0) & (idx < 12)).all())


# ------------------------------------------------------------------------------------------------ norms
@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("W", [44, 45, 256, 3000, 4096])
def test_sandwich_norm(W, device, dtype):
    g = torch.Generator().manual_seed(W)
    T, k, eps = 5, 3, 1e-4
    x, add = torch.randn(T, W, generator=g) * 3, torch.randn(T, W, generator=g)
    y, wp, wn = (torch.randn(*s, generator=g).to(dtype) for s in ((T * k, W), (W,), (W,)))
    slots = torch.randperm(T * k, generator=g).view(T, k).to(torch.int32)
    index = torch.tensor([4, 0, 4])
    dev = [t.to(device) for t in (x, y, wp, wn, add, slots, index)]
    tol = 1e-2 if dtype == torch.bfloat16 else 1e-5
    for use_slots in (False, True):
        for use_add in (False, True):
            for use_index in (False, True):
                yy = y.double()[slots.long()].sum(1) if use_slots else y.double()[:T]
                o = x.double() + O.rms_norm(yy, wp.double(), eps) + (add.double() if use_add else 0)
                o = o[index] if use_index else o
                gx, gh = RN.sandwich_norm(dev[0], dev[1] if use_slots else dev[1][:T], dev[2], dev[3], eps, dev[5] if use_slots else None,
                                          dev[4] if use_add else None, dev[6] if use_index else None)
                close(gx, o, 1e-5)
                close(gh, O.rms_norm(o, wn.double(), eps), tol)
                assert gx.dtype == torch.float32 and gh.dtype == dtype


@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("W", [44, 45, 1024])
def test_embed_and_gated_norm(W, device, dtype):
    g = torch.Generator().manual_seed(W)
    table, w, wn, x, gate = (torch.randn(*s, generator=g).to(dtype) for s in ((9, W), (W,), (W,), (4, W), (4, 2 * W + 8)))
    ids = torch.tensor([3, 8, 0, 3])
    tol = 1e-2 if dtype == torch.bfloat16 else 1e-5
    gx, gh = RN.embed_norm(table.to(device), ids.to(device), w.to(device), 1e-3, wn.to(device))
    ref = O.rms_norm(table.double()[ids], w.double(), 1e-3)
    close(gx, ref, 1e-5)
    close(gh, O.rms_norm(ref, wn.double(), 1e-3), tol)
    go = RN.gated_rms_norm(x.to(device), w.to(device), gate.to(device)[:, 8:8 + W], 1e-3)
    close(go, O.rms_norm(x.double(), w.double(), 1e-3) * torch.sigmoid(gate.double()[:, 8:8 + W]), tol)


# ------------------------------------------------------------------------------- fused decode launches
@gpu
@pytest.mark.parametrize("M,K,N", [(1, 4096, 96), (2, 4096, 48), (4, 2048, 4096), (3, 72, 24), (1, 8192, 32), (2, 256, 8192)])
def test_fused_sandwich_launches(M, K, N):
    from shuffle_exchange_amd.ops import linear as LI
    g = torch.Generator().manual_seed(K)
    k, eps, E = 3, 1e-4, 11
    x, add = torch.randn(M, K, generator=g) * 3, torch.randn(M, K, generator=g)
    y, wp, wn, w, router = (torch.randn(*s, generator=g).to(torch.bfloat16) for s in ((M * k, K), (K,), (K,), (N, K), (E, K)))
    slots = torch.randperm(M * k, generator=g).view(M, k).to(torch.int32)
    xd, yd, wpd, wnd, wd, rd, ad, sd = (t.cuda() for t in (x, y, wp, wn, w, router, add, slots))
    for use_slots in (False, True):
        for use_add in (False, True):
            yy = y.double()[slots.long()].sum(1) if use_slots else y.double()[:M]
            v = x.double() + O.rms_norm(yy, wp.double(), eps) + (add.double() if use_add else 0)
            h = O.rms_norm(v, wn.double(), eps)
            args = (xd, yd if use_slots else yd[:M], wpd, wnd, eps, sd if use_slots else None, ad if use_add else None)
            out, gx = LI.fused_sandwich_linear(*args, wd)
            close(gx, v, 1e-5)
            close(out, h @ w.double().T, 2e-2)
            gx, gh, routing = ME.fused_sandwich_route(*args, rd, 4)
            close(gx, v, 1e-5)
            close(gh, h, 1e-2)
            val, idx = (gh.double().cpu() @ router.double().T).topk(4, dim=-1)
            assert torch.equal(routing.expert.cpu().long(), idx)
            torch.testing.assert_close(routing.weight.double().cpu(), torch.softmax(val, -1), rtol=1e-4, atol=1e-6)
    assert LI.fused_sandwich_linear(torch.zeros(2, 8192, device="cuda"), torch.zeros(2, 8192, device="cuda").bfloat16(),
                                    wpd.new_ones(8192), wpd.new_ones(8192), eps, None, None, wpd.new_ones(8, 8192)) is None
    gate = torch.randn(M, K + 16, generator=g).to(torch.bfloat16)
    out = LI.fused_gatenorm_linear(yd[:M], wpd, gate.cuda()[:, 16:], eps, wd)
    close(out, (O.rms_norm(y.double()[:M], wp.double(), eps) * torch.sigmoid(gate.double()[:, 16:])) @ w.double().T, 2e-2)
