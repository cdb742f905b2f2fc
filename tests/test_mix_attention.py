"""ops/mix_attention.py and ops/residual_norm.py against the plain functions of tobinex_oracle.py: the
PyTorch forms on the CPU, every HIP form on the GPU."""
import itertools
import os
import sys
import types

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import tobinex_oracle as O  # noqa: E402
from shuffle_exchange_amd.ops.mix_attention import MixParams, cache_row, mix_attention  # noqa: E402
from shuffle_exchange_amd.ops.residual_norm import embed_scale, qkv_norm_append, residual_rms_norm  # noqa: E402

gpu = pytest.mark.gpu


class Case:
    """Ragged sequences over a paged cache with shuffled blocks; ``lens`` = (history, new tokens)."""

    def __init__(self, lens, H, G, dk, dv, dtype, device, bs=32, seed=0, garbage=True):
        g = torch.Generator().manual_seed(seed)
        self.lens, self.H, self.G, self.dk, self.dv, self.dtype = lens, H, G, dk, dv, dtype
        S = len(lens)
        self.rows = (cache_row(dk, dtype), cache_row(dv, dtype))
        if dtype == torch.bfloat16:
            self.rows = (max(self.rows),) * 2
        tot = [a + n for a, n in lens]
        nb = [(t + bs - 1) // bs for t in tot]
        perm = torch.randperm(sum(nb) + 3, generator=g)
        # blocks hold finite leftovers of earlier sequences
        kc, vc = ((torch.randn(sum(nb) + 3, G, bs, r, generator=g) * (3.0 if garbage else 0.0)) for r in self.rows)
        bt = torch.zeros(S, max(nb), dtype=torch.int32)
        self.k, self.v, self.q, at = [], [], [], 0
        for s, (a, n) in enumerate(lens):
            k, v = torch.randn(tot[s], G, dk, generator=g), torch.randn(tot[s], G, dv, generator=g)
            k, v = k.to(dtype).float(), v.to(dtype).float()
            self.k.append(k)
            self.v.append(v)
            self.q.append(torch.randn(n, H, dk, generator=g).to(dtype).float())
            for b in range(nb[s]):
                blk = int(perm[at])
                at += 1
                bt[s, b] = blk
                m = min(bs, tot[s] - b * bs)
                for c, x, d in ((kc, k, dk), (vc, v, dv)):
                    c[blk, :, :m] = 0
                    c[blk, :, :m, :d] = x[b * bs:b * bs + m].transpose(0, 1)
        self.q_pad = torch.zeros(sum(n for _, n in lens), H, self.rows[0])
        self.q_pad[..., :dk] = torch.cat(self.q)
        self.p = MixParams(torch.rand(H, generator=g) * 1.5, torch.rand(H, generator=g) * 0.5,
                           torch.randn(H, generator=g) + 1.0,
                           (torch.eye(H) + torch.randn(H, H, generator=g) * H ** -0.5).to(torch.bfloat16).float())
        self.gate = torch.randn(self.q_pad.shape[0], H * dv, generator=g).to(dtype)
        self.device, self.bt, self.kc, self.vc = device, bt, kc, vc

    def batch(self):
        i32 = (lambda x: torch.tensor(x, dtype=torch.int32, device=self.device))
        ql = [n for _, n in self.lens]
        kl = [a + n for a, n in self.lens]
        return types.SimpleNamespace(block_table=self.bt.to(self.device), q_start=i32([sum(ql[:i]) for i in range(len(ql))]),
                                     q_len=i32(ql), kv_len=i32(kl), host_q_len=ql, max_kv_len=max(kl), num_seqs=len(ql))

    def run(self, scale, window, keep, form="auto", use=("bias", "sink", "talk", "gate")):
        d = (lambda t: t.to(self.device))
        p = MixParams(*(d(x) if n in use else None for x, n in
                        ((self.p.r1, "bias"), (self.p.r2, "bias"), (self.p.sink, "sink"), (self.p.talk, "talk"))))
        return mix_attention(d(self.q_pad.to(self.dtype)), d(self.kc.to(self.dtype)), d(self.vc.to(self.dtype)), self.batch(),
                             self.dk, self.dv, scale, p, window, keep, gate=d(self.gate) if "gate" in use else None,
                             form=form).float().cpu()

    def oracle(self, scale, window, keep, use=("bias", "sink", "talk", "gate")):
        """(output, sqrt(sum_j (w v)^2)): what rounding of the weights to bf16 is relative to -- plus a hundredth
        of the same with |talk|, for mixed weights that nearly cancel."""
        outs, mags, kv = [], [], torch.arange(self.H) // (self.H // self.G)
        for q, k, v, (a, n) in zip(self.q, self.k, self.v, self.lens):
            T = a + n
            qq, kk, vv = (x.double().transpose(0, 1) for x in (torch.cat([torch.zeros(a, *q.shape[1:]), q]), k, v))
            s = qq @ kk[kv].transpose(1, 2) * scale
            if "bias" in use:
                s = s - O.distance_bias(self.p.r1.double(), self.p.r2.double(), T)
            sink = self.p.sink.double() if "sink" in use else torch.full((self.H,), -1e30, dtype=torch.float64)
            w = O.sink_softmax(s, O.window_mask(T, window, keep), sink)
            floor = O.talking_heads(w, self.p.talk.double().abs()) if "talk" in use else w
            if "talk" in use:
                w = O.talking_heads(w, self.p.talk.double())
            outs.append((w @ vv[kv]).transpose(0, 1).reshape(T, -1)[a:])
            mags.append((((w * w) @ (vv * vv)[kv]).sqrt() + 0.01 * ((floor * floor) @ (vv * vv)[kv]).sqrt())
                       .transpose(0, 1).reshape(T, -1)[a:])
        g = torch.sigmoid(self.gate.double()) if "gate" in use else 1.0
        return (torch.cat(outs) * g).float(), (torch.cat(mags) * g).float()


def check(got, ref, dtype, rows=slice(None)):
    tol = 2e-5 if dtype == torch.float32 else 0.012
    o, mag = ref
    err = ((got - o).abs() / (o.abs() + mag))[rows]
    assert float(err.max()) < tol, f"max error {float(err.max()):.3e}"


LENS = [(0, 70), (37, 1), (0, 1), (100, 3), (31, 33), (64, 9)]


@pytest.mark.parametrize("window,keep", [(None, 0), (24, 5), (1, 0), (16, 40), (200, 3)])
def test_cpu_form(window, keep):
    c = Case(LENS, 6, 2, 20, 12, torch.float32, "cpu")
    check(c.run(0.3, window, keep), c.oracle(0.3, window, keep), torch.float32)


@pytest.mark.parametrize("use", [(), ("bias",), ("sink",), ("talk",), ("gate",)])
def test_cpu_form_each_mechanism(use):
    c = Case([(0, 20), (9, 5)], 4, 4, 8, 8, torch.float32, "cpu")
    check(c.run(0.5, 7, 2, use=use), c.oracle(0.5, 7, 2, use=use), torch.float32)


SIZES = [(6, 2, 20, 12), (8, 8, 64, 64), (4, 1, 40, 72), (1, 1, 16, 16), (12, 4, 48, 24), (5, 5, 33, 7)]


@gpu
@pytest.mark.parametrize("H,G,dk,dv", SIZES)
def test_generic_fp32(H, G, dk, dv):
    for window, keep in ((None, 0), (24, 5), (16, 40)):
        c = Case(LENS, H, G, dk, dv, torch.float32, "cuda")
        check(c.run(dk ** -0.5, window, keep), c.oracle(dk ** -0.5, window, keep), torch.float32)


@gpu
@pytest.mark.parametrize("form", ["generic", "token", "tile", "auto"])
@pytest.mark.parametrize("H,G,dk,dv", SIZES + [(32, 8, 128, 128), (16, 4, 128, 96), (32, 4, 64, 64), (24, 8, 64, 64),
                                               (32, 16, 128, 128), (20, 20, 64, 64), (17, 1, 128, 128)])
def test_forms_bf16(form, H, G, dk, dv):
    for window, keep in ((None, 0), (24, 5), (1, 0), (16, 40), (64, 1)):
        c = Case(LENS, H, G, dk, dv, torch.bfloat16, "cuda", seed=H)
        check(c.run(dk ** -0.5, window, keep, form), c.oracle(dk ** -0.5, window, keep), torch.bfloat16)


@gpu
@pytest.mark.parametrize("form", ["generic", "token", "auto"])
@pytest.mark.parametrize("H,G,dk,dv", [(40, 8, 64, 64), (48, 2, 128, 128), (8, 2, 256, 256), (4, 2, 192, 128), (96, 4, 32, 32)])
def test_large_heads_bf16(form, H, G, dk, dv):
    for window, keep in ((None, 0), (24, 5)):
        c = Case(LENS, H, G, dk, dv, torch.bfloat16, "cuda", seed=H)
        check(c.run(dk ** -0.5, window, keep, form), c.oracle(dk ** -0.5, window, keep), torch.bfloat16)


@gpu
@pytest.mark.parametrize("form", ["generic", "token", "tile"])
@pytest.mark.parametrize("use", [(), ("bias",), ("sink",), ("talk",), ("gate",), ("bias", "talk")])
def test_each_mechanism_bf16(form, use):
    c = Case(LENS, 8, 4, 64, 64, torch.bfloat16, "cuda")
    check(c.run(0.125, 20, 6, form, use), c.oracle(0.125, 20, 6, use), torch.bfloat16)


@gpu
@pytest.mark.parametrize("form", ["generic", "token", "tile"])
def test_window_edges_stand_out(form):
    """One key just inside and one just outside the window, and the last kept / first dropped early key,
    each made to stand out for the query: the output must follow the mask exactly."""
    W, keep = 32, 5
    for pos, key in itertools.product((96, 97, 127, 128), ("in", "out", "kept", "dropped")):
        n = pos + 1
        j = {"in": pos - W + 1, "out": pos - W, "kept": keep - 1, "dropped": keep}[key]
        c = Case([(0, n), (pos, 1)], 8, 2, 64, 64, torch.bfloat16, "cuda", seed=pos)
        for s in range(2):
            c.q[s][-1] = c.k[s][j].repeat_interleave(4, 0) * 2
        c.q_pad[n - 1, :, :64], c.q_pad[n, :, :64] = c.q[0][-1], c.q[1][-1]
        check(c.run(0.125, W, keep, form), c.oracle(0.125, W, keep), torch.bfloat16, [n - 1, n])


@gpu
def test_many_splits_and_long_context():
    c = Case([(3000, 1), (700, 1), (5, 1)], 16, 4, 128, 128, torch.bfloat16, "cuda", bs=64)
    for window, keep in ((None, 0), (1500, 70)):
        check(c.run(0.09, window, keep), c.oracle(0.09, window, keep), torch.bfloat16)


@gpu
def test_tile_form_key_splits_and_many_tiles():
    for lens, H, G, D in (([(0, 700)], 32, 8, 64), ([(1400, 90), (0, 20)], 16, 4, 128), ([(0, 2300)], 4, 2, 64)):
        c = Case(lens, H, G, D, D, torch.bfloat16, "cuda", bs=64)
        for window, keep in ((None, 0), (600, 50)):
            check(c.run(0.1, window, keep, "tile"), c.oracle(0.1, window, keep), torch.bfloat16)


# ------------------------------------------------------------------------------------- row ops
def _row_case(W, dtype, device):
    g = torch.Generator().manual_seed(W)
    x, y = torch.randn(9, W, generator=g), torch.randn(9, W, generator=g).to(dtype)
    w = (torch.randn(W, generator=g) * 0.3).to(dtype)
    return x.to(device), y.to(device), w.to(device)


def _check_rows(W, dtype, device):
    x, y, w = _row_case(W, dtype, device)
    ref = O.norm_around_zero(2.5 * x.double().cpu() + y.double().cpu(), w.double().cpu(), 1e-3)
    o, ob = residual_rms_norm(x, y, w, 2.5, 1e-3, 1.0)
    assert o.dtype == torch.float32 and ob.dtype == dtype
    torch.testing.assert_close(o.double().cpu(), ref, rtol=2e-6, atol=2e-6)
    torch.testing.assert_close(ob.double().cpu(), ref, rtol=5e-3, atol=5e-3)
    idx = torch.tensor([8, 0, 3], device=device)
    _, pb = residual_rms_norm(x, None, w, 1.0, 1e-3, 0.0, index=idx, need_x=False)
    ref = O.projection_norm(x.double().cpu()[[8, 0, 3]], w.double().cpu(), 1e-3)
    torch.testing.assert_close(pb.double().cpu(), ref, rtol=5e-3, atol=5e-3)
    table = torch.randn(11, W).to(dtype).to(device)
    e, eb = embed_scale(table, torch.tensor([10, 0, 4], device=device), 12.0)
    torch.testing.assert_close(e.cpu(), table.float().cpu()[[10, 0, 4]] * 12.0)
    torch.testing.assert_close(eb.cpu(), e.to(dtype).cpu())


@pytest.mark.parametrize("W", [64, 100])
def test_rows_cpu(W):
    _check_rows(W, torch.float32, "cpu")


@gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W", [64, 250, 1024, 1028, 5000, 9001, 20000])
def test_rows_gpu(W, dtype):
    _check_rows(W, dtype, "cuda")


def _check_append(nq, nkv, dk, dv, dtype, device):
    g = torch.Generator().manual_seed(nq)
    T, bs = 7, 16
    extra = 5
    proj = torch.randn(T, nq * dk + nkv * (dk + dv) + extra, generator=g).to(dtype).to(device)
    qw, kw = ((torch.rand(n, generator=g) + 0.5).to(dtype).to(device) for n in (nq * dk, nkv * dk))
    D = max(cache_row(dk, dtype), cache_row(dv, dtype)) if dtype == torch.bfloat16 else None
    Dk, Dv = (D, D) if D else (dk, dv)
    kc, vc = (torch.full((4, nkv, bs, d), 9.0, dtype=dtype, device=device) for d in (Dk, Dv))
    slots = torch.tensor([3, 17, 63, 16, -1, 0, 48], device=device)
    q = qkv_norm_append(proj, qw, kw, kc, vc, slots, nq, nkv, dk, dv, 1e-4).double().cpu()
    P = proj.double().cpu()
    a, b = nq * dk, nq * dk + nkv * dk
    tol = dict(rtol=2e-6, atol=2e-6) if dtype == torch.float32 else dict(rtol=5e-3, atol=5e-3)
    ref_q = O.projection_norm(P[:, :a], qw.double().cpu(), 1e-4).view(T, nq, dk)
    torch.testing.assert_close(q[..., :dk], ref_q, **tol)
    assert not q[..., dk:].any()
    ref_k = O.projection_norm(P[:, a:b], kw.double().cpu(), 1e-4).view(T, nkv, dk)
    ref_v = P[:, b:b + nkv * dv].view(T, nkv, dv)
    seen = torch.zeros(4, bs, dtype=torch.bool)
    for t, s in enumerate(slots.tolist()):
        if s < 0:
            continue
        seen[s // bs, s % bs] = True
        for c, r, d in ((kc, ref_k, dk), (vc, ref_v, dv)):
            torch.testing.assert_close(c[s // bs, :, s % bs, :d].double().cpu(), r[t], **tol)
            assert not c[s // bs, :, s % bs, d:].any()
    assert bool((kc.transpose(1, 2).cpu()[~seen] == 9).all()) and bool((vc.transpose(1, 2).cpu()[~seen] == 9).all())


@pytest.mark.parametrize("shape", [(6, 2, 20, 12), (4, 4, 8, 8)])
def test_append_cpu(shape):
    _check_append(*shape, torch.float32, "cpu")


@gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("shape", [(6, 2, 20, 12), (8, 8, 64, 64), (32, 8, 128, 128), (3, 1, 40, 72), (5, 5, 33, 7)])
def test_append_gpu(shape, dtype):
    _check_append(*shape, dtype, "cuda")


# --------------------------------------------------------------------------- fused decode projections
@gpu
@pytest.mark.parametrize("M", [1, 3, 4])
@pytest.mark.parametrize("K,N", [(64, 48), (256, 1000), (4096, 4096), (1048, 40)])
def test_fused_addnorm_and_gatesum(M, K, N):
    from shuffle_exchange_amd.ops.linear import fused_addnorm_linear, fused_gatesum_linear
    g = torch.Generator().manual_seed(K + M)
    bf = (lambda *s, std=1.0: (torch.randn(*s, generator=g) * std).to(torch.bfloat16).cuda())
    w1, w2 = bf(N, K, std=K ** -0.5), bf(N, K, std=K ** -0.5)
    y1, y2, n1, n2 = bf(M, K), bf(M, K), bf(K, std=0.3), bf(K, std=0.3)
    x = torch.randn(M, K, generator=g).cuda()
    o1, st = fused_addnorm_linear(y1, x, n1, 2.0, 1e-3, 1.0, w1)
    o2, st2 = fused_addnorm_linear(y2, st, n2, 2.0, 1e-3, 1.0, w2)
    d = (lambda t: t.double().cpu())
    r1 = O.norm_around_zero(2.0 * d(x) + d(y1), d(n1), 1e-3)
    r2 = O.norm_around_zero(2.0 * r1 + d(y2), d(n2), 1e-3)
    for o, r, w in ((o1, r1, w1), (o2, r2, w2)):
        torch.testing.assert_close(d(o), r @ d(w).T, rtol=2e-2, atol=3e-2)
    torch.testing.assert_close(d(st2[0]), 2.0 * r1 + d(y2), rtol=1e-5, atol=1e-5)
    stream = residual_rms_norm(st2[0], None, n2, 1.0, 1e-3, 1.0)[0]
    torch.testing.assert_close(d(stream), r2, rtol=1e-5, atol=1e-5)
    torch.testing.assert_close(d(stream), d(st2[0]) * d(st2[1])[:, None] * (1 + d(n2)), rtol=1e-5, atol=1e-5)
    for splits in (1, 3, 11):
        part, gate = torch.randn(splits, M, K, generator=g).cuda(), bf(M, K + 8)[:, 8:]
        ref = (d(part).sum(0) * torch.sigmoid(d(gate))) @ d(w1).T
        torch.testing.assert_close(d(fused_gatesum_linear(part, gate, w1)), ref, rtol=2e-2, atol=0.02 * splits ** 0.5 + 0.02)
