"""Topelorn on the GPU: its kernels one by one against fp32 PyTorch, the model in
32 and 16 bits against the slow oracle under every way of cutting and batching,
generation through the scheduler, the trace command."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import mcp_amd.ops as ops
from mcp_amd.engine.batch import BLOCK_SIZE, StepInputs, long_spans, pack
from mcp_amd.models import topelorn
from mcp_amd.models.llama import padded_group
from mcp_amd.ops import reference as ref

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import topelorn_cases as cases  # noqa: E402
import topelorn_oracle as oracle  # noqa: E402
from test_masked_attention_gpu import _case  # noqa: E402

pytestmark = pytest.mark.gpu
DEV = "cuda"
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _rnd(*shape, seed=0, dtype=torch.float32, scale=1.0):
    g = torch.Generator(device=DEV).manual_seed(seed)
    return (torch.randn(*shape, generator=g, device=DEV) * scale).to(dtype)


def _close(got, want, tol):
    err = (got.double() - want.double()).abs().max() / want.double().abs().max().clamp(min=1e-9)
    assert err < tol, float(err)


# ------------------------------------------------------------------- kernels
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("rows,H,Hp", [(1, 100, 128), (3, 320, 320), (700, 199, 256), (1, 4096, 4096),
                                       (5, 5000, 5056), (600, 8192, 8192), (2, 16384, 16384)])
def test_layer_norm_with_plain_add(rows, H, Hp, dtype):
    def padded(t):
        t[..., H:] = 0
        return t
    x, y = padded(_rnd(rows, Hp, seed=1) + 4.0), padded(_rnd(rows, Hp, seed=2, scale=3.0)).to(dtype)
    w = padded(_rnd(Hp, seed=3))
    for kw in (dict(y=y, w_pre=w), dict(w_pre=w), dict(y=y)):
        gx, wx = x.clone(), x.clone()
        out = None if "w_pre" not in kw else torch.empty_like(y)
        got = ops.residual_norm(gx, H, 1e-5, out=out, center=True, **kw)
        want = ref.residual_norm(wx, H, 1e-5, out=None if out is None else torch.empty_like(y), center=True, **kw)
        assert torch.equal(gx, wx)
        if out is not None:
            _close(got, want, 1e-5 if dtype == torch.float32 else 8e-3)
            assert not got[:, H:].any()


@pytest.mark.parametrize("M,N,K", [(1, 4, 64), (65, 452, 320)])
def test_gemm_f32_residual(M, N, K):
    X, W, R = _rnd(M, K, seed=1), _rnd(N, K, seed=2), _rnd(M, N, seed=3)
    _close(ops.gemm(X, W, R=R), X.double() @ W.double().t() + R, 2e-6)


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("T", [1, 3, 16, 17, 33, 64, 65, 130, 300])
@pytest.mark.parametrize("H,N,K", [(1, 16, 32), (3, 80, 96), (5, 128, 64), (2, 512, 128), (4, 144, 576)])
def test_gemm_heads(T, H, N, K, dtype):
    """Strided views in, strided views out, nothing outside them written."""
    z = _rnd(T, H * (K + 16) + 24, seed=1, dtype=dtype)
    X = z[:, 8:8 + H * (K + 16)].view(T, H, K + 16)[..., 8:8 + K]
    W = _rnd(H, N, K, seed=2, dtype=dtype)
    wide = torch.full((T, H, N + 48), 7.0, device=DEV, dtype=dtype)
    ops.gemm_heads(X, W, wide[..., 16:16 + N])
    want = torch.stack([X[:, h].float() @ W[h].float().t() for h in range(H)], 1)
    _close(wide[..., 16:16 + N].float(), want, 1e-2 if dtype == torch.bfloat16 else 2e-6)
    assert (wide[..., :16] == 7).all() and (wide[..., 16 + N:] == 7).all()


def _slots(T, nb, seed=5):
    slots = torch.randperm(nb * 64, generator=torch.Generator().manual_seed(seed))[:T].int()
    if T > 1:
        slots[T // 2] = -1
    return slots


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("T", [1, 37, 200])
@pytest.mark.parametrize("Hq,Hkv,DK,DV,dim", [(6, 2, 64, 64, 40), (4, 4, 128, 64, 128), (5, 1, 64, 192, 24),
                                              (2, 1, 256, 256, 250), (2, 2, 320, 576, 300), (1, 1, 768, 64, 700)])
def test_qk_norm_kv(T, Hq, Hkv, DK, DV, dim, dtype):
    cols = (Hq + Hkv) * DK + Hkv * DV
    z = _rnd(T, cols + 16, seed=1, dtype=dtype)
    z[:, :(Hq + Hkv) * DK].view(T, Hq + Hkv, DK)[..., dim:] = 0
    wq, wk = _rnd(DK, seed=2), _rnd(DK, seed=3)
    first = _rnd(T, 2 * Hkv * DV, seed=4, dtype=dtype)[:, Hkv * DV:]
    nb = T // 64 + 2
    slots = _slots(T, nb)
    for mix in (None, first):
        def run(f, dev, dt, zz, v1, w1, w2):
            q = torch.zeros(T, Hq, DK, device=dev, dtype=dt)
            kc = torch.zeros(nb, Hkv, 64, DK, device=dev, dtype=dt)
            vc = torch.zeros(nb, Hkv, 64, DV, device=dev, dtype=dt)
            f(zz, slots.to(dev), w1, w2, dim, 1e-3, q, kc, vc, v1, 0.3)
            return q, kc, vc
        got = run(ops.qk_norm_kv, DEV, dtype, z, mix, wq, wk)
        want = run(ref.qk_norm_kv, "cpu", torch.float32, z.float().cpu(), None if mix is None else mix.float().cpu(),
                   wq.cpu(), wk.cpu())
        for g, w in zip(got, want):
            _close(g.cpu().float(), w, 8e-3 if dtype == torch.bfloat16 else 1e-5)


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("T", [1, 70])
@pytest.mark.parametrize("H,dim,rot,rank,n,pairs,DK", [(3, 32, 32, 96, 90, 16, 128), (2, 64, 16, 48, 48, 6, 64),
                                                       (32, 128, 64, 512, 512, 32, 576), (1, 32, 16, 1008, 1000, 0, 1024)])
def test_latent_qkv(T, H, dim, rot, rank, n, pairs, DK, dtype):
    cols = H * (dim + rot) + rank + rot
    z = _rnd(T, cols + 16, seed=1, dtype=dtype)
    z[:, H * (dim + rot) + n:H * (dim + rot) + rank] = 0
    w_c = _rnd(rank, seed=2)
    pos = torch.randint(0, 400, (T,), generator=torch.Generator().manual_seed(4)).int()
    cs = torch.randn(400, pairs, 2, generator=torch.Generator().manual_seed(6))
    nb = T // 64 + 2
    slots = _slots(T, nb)

    def run(f, dev, dt, zz):
        q, kc = torch.full((T, H, DK), 3.0, device=dev, dtype=dt), torch.zeros(nb, 1, 64, DK, device=dev, dtype=dt)
        f(zz, pos.to(dev), slots.to(dev), cs.to(dev), w_c.to(dev), 1e-3, H, dim, rot, rank, n, q, kc)
        return q, kc
    for g, w in zip(run(ops.latent_qkv, DEV, dtype, z), run(ref.latent_qkv, "cpu", torch.float32, z.float().cpu())):
        _close(g.cpu().float(), w, 8e-3 if dtype == torch.bfloat16 else 1e-5)
    kc = torch.zeros(nb, 1, 64, DK, device=DEV, dtype=dtype)
    ops.latent_qkv(z, pos.to(DEV), slots.to(DEV), cs.to(DEV), w_c, 1e-3, H, dim, rot, rank, n, None, kc)
    assert torch.equal(kc, run(ops.latent_qkv, DEV, dtype, z)[1])


# ----------------------------------------------------------------- attention
MIXED = [(0, 70), (63, 1), (64, 1), (190, 3), (0, 1), (129, 40), (255, 2), (400, 9)]


def _check(spans, Hq, Hkv, DK, DV, window, keep, slopes=True, sinks=True, gate=True, dtype=torch.bfloat16,
           splits=1, seed=0, amp=1.0, shared=False):
    q, kc, vc, step = _case(spans, Hq, Hkv, DK, DV, dtype, seed, amp=amp)
    group = padded_group(min(Hq // Hkv, 16))
    dev = pack(step, group, DEV)
    dev.attn.kv_splits = splits
    g = torch.Generator().manual_seed(seed + 1)
    T, scale = q.shape[0], DK ** -0.5
    kw = dict(window=window, keep_first=keep)
    if slopes:
        kw["slopes"] = torch.tensor([oracle.slope(h, Hq) for h in range(Hq)])
    if sinks:
        kw["sink"] = torch.randn(Hq, generator=g) * 2
    gates = torch.randn(T, Hq + 5, generator=g).to(dtype)
    put = lambda v: v.to(DEV) if isinstance(v, torch.Tensor) else v  # noqa: E731
    got = ops.masked_attention(q.to(DEV), kc.to(DEV), None if shared else vc.to(DEV), dev.attn, scale, group,
                               gate=gates.to(DEV)[:, 3:3 + Hq] if gate else None, v_dim=DV if shared else None,
                               **{k: put(v) for k, v in kw.items()})
    t = lambda a: torch.from_numpy(np.asarray(a))  # noqa: E731
    want = ref.masked_attention(q.float(), kc.float().nan_to_num(), None if shared else vc.float().nan_to_num(),
                                t(step.q_start), t(step.q_len), t(step.ctx_len), t(step.block_table), scale,
                                gate=gates.float()[:, 3:3 + Hq] if gate else None, v_dim=DV if shared else None, **kw)
    assert torch.isfinite(got).all()
    err = (got.float().cpu() - want).abs().amax(dim=(1, 2)) / want.abs().amax()
    assert err.max() < (3e-5 if dtype == torch.float32 else 1.2e-2), (float(err.max()), int(err.argmax()))


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("Hq,Hkv,DK,DV", [(6, 2, 64, 64), (8, 2, 128, 128), (6, 2, 128, 64), (5, 5, 64, 128),
                                          (40, 2, 64, 64), (7, 1, 192, 128), (4, 2, 256, 256), (3, 1, 320, 64)])
def test_windowed_head_shapes(Hq, Hkv, DK, DV, dtype):
    _check(MIXED, Hq, Hkv, DK, DV, 75, 9, dtype=dtype)


@pytest.mark.parametrize("window", [0, 1, 2, 63, 64, 65, 100, 128, 5000])
@pytest.mark.parametrize("keep", [0, 1, 64, 70, 200])
def test_windows_and_kept_tokens(window, keep):
    _check(MIXED, 8, 2, 128, 128, window, keep, amp=2.0, seed=window)
    _check(MIXED, 8, 2, 128, 128, window, keep, slopes=False, sinks=False, gate=False, seed=keep)


@pytest.mark.parametrize("splits", [2, 8, 32])
@pytest.mark.parametrize("window,keep", [(0, 0), (700, 5), (129, 130)])
def test_windows_with_split_keys(splits, window, keep):
    spans = [(1500, 1), (70, 1), (0, 2), (999, 3), (640, 1)]
    _check(spans, 8, 2, 128, 128, window, keep, splits=splits)
    _check(spans, 6, 2, 64, 128, window, keep, slopes=False, splits=splits, amp=2.0)


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("DK,DV", list(ops.LATENT_SIZES) + [(640, 576)])
@pytest.mark.parametrize("Hq", [1, 3, 16, 20, 33, 70])
def test_latent_shapes(DK, DV, Hq, dtype):
    _check(MIXED[:6], Hq, 1, DK, DV, 75, 0, slopes=False, sinks=False, dtype=dtype, shared=True)


@pytest.mark.parametrize("window", [0, 1, 2, 63, 64, 65, 128, 5000])
@pytest.mark.parametrize("splits", [1, 8])
def test_latent_windows(window, splits):
    _check(MIXED, 20, 1, 192, 128, window, 0, slopes=False, sinks=False, seed=window, splits=splits, amp=2.0, shared=True)
    _check([(1500, 1), (70, 1), (0, 2), (999, 6), (640, 1)], 40, 1, 576, 512, window, 0, slopes=False, sinks=False,
           seed=window, splits=splits, shared=True)
    _check([(900, 17), (700, 1), (800, 12)], 24, 1, 320, 256, window, 0, slopes=False, sinks=False, splits=splits,
           shared=True)
    _check(MIXED, 8, 1, 128, 64, max(window, 1), 3, slopes=False, seed=window, splits=splits, shared=True)


@pytest.mark.parametrize("window", [100, 128, 192])
@pytest.mark.parametrize("shared", [False, True])
def test_window_edges_stand_out(window, shared):
    """One huge key just inside, one just outside the window and the kept keys: a
    mask that is one position off changes the output completely."""
    keep = 5
    for pos in (window + keep - 1, window + keep, 2 * window - 1, 2 * window + 63):
        for new in (1, 2, 5, 60, pos + 1):
            # (the first 64 columns of a key are its value in the shared form: scores use the others)
            q, kc, vc, step = _case([(pos + 1 - new, new)], 2, 1, 128, 64, torch.bfloat16, seed=pos)
            bt = step.block_table[0]
            u = torch.randn(64, generator=torch.Generator().manual_seed(pos))
            u = (u / u.norm() * 16).to(torch.bfloat16)
            q[-1, :, :64], q[-1, :, 64:] = 0, u
            for inside in (pos - window + 1, keep - 1):
                k2, v2 = kc.clone(), vc.clone()
                outside = [j for j in (pos - window, keep) if keep <= j <= pos - window]
                for key, v in [(inside, 3.0)] + [(j, -50.0) for j in outside]:
                    k2[bt[key // 64], 0, key % 64, 64:] = u
                    k2[bt[key // 64], 0, key % 64, :64] = v
                    v2[bt[key // 64], 0, key % 64] = v
                dev = pack(step, 2, DEV)
                got = ops.masked_attention(q.to(DEV), k2.to(DEV), None if shared else v2.to(DEV), dev.attn, 0.125, 2,
                                           window=window, keep_first=keep, v_dim=64 if shared else None)[-1].float()
                assert (got - 3.0).abs().max() < 0.06, (pos, new, inside)


def test_split_and_gate_rows_do_not_depend_on_the_batch():
    spans = [(130, 1), (0, 90), (77, 5)]
    for shared, (Hq, Hkv, DK, DV) in ((False, (8, 2, 128, 128)), (True, (20, 1, 192, 128))):
        q, kc, vc, step = _case(spans, Hq, Hkv, DK, DV, torch.bfloat16, seed=3)
        gates = _rnd(q.shape[0], Hq, dtype=torch.bfloat16)
        k = dict(window=100, keep_first=2, sink=_rnd(Hq), v_dim=DV if shared else None)
        vd = None if shared else vc.to(DEV)
        alls = ops.masked_attention(q.to(DEV), kc.to(DEV), vd, pack(step, 4, DEV).attn, 0.09, 4, gate=gates, **k)
        for i, (c, n) in enumerate(spans):
            a = int(step.q_start[i])
            one = StepInputs(np.zeros(n, np.int32), np.zeros(n, np.int32), np.zeros(n, np.int32),
                             np.zeros(1, np.int32), step.q_len[i:i + 1], step.ctx_len[i:i + 1],
                             step.block_table[i:i + 1], np.zeros(0, np.int32))
            alone = ops.masked_attention(q[a:a + n].to(DEV).contiguous(), kc.to(DEV), vd, pack(one, 4, DEV).attn, 0.09,
                                         4, gate=gates[a:a + n], **k)
            assert torch.equal(alone, alls[a:a + n])


@pytest.mark.parametrize("H,dim,rot,rot_dims,rank,vdim,window", [
    (4, 128, 64, 64, 512, 128, 0), (4, 128, 64, 64, 512, 128, 150), (3, 32, 32, 32, 48, 64, 64), (2, 64, 16, 12, 96, 192, 65),
    (1, 96, 16, 0, 112, 64, 300), (2, 160, 64, 64, 64, 256, 1)])
def test_long_spans_on_expanded_latents(H, dim, rot, rot_dims, rank, vdim, window):
    """The expanded form against plain attention on the projected keys; other
    spans' rows stay as they are; pages hold stale NaN past the last key."""
    spans = [(0, 300), (40, 3), (130, 256), (500, 257), (70, 1)]
    _, kc, _, step = _case(spans, 1, 1, ops_row(rank, rot), 64, torch.bfloat16, seed=window)
    T = sum(n for _, n in spans)
    z = _rnd(T, H * (dim + rot) + 16, seed=1, dtype=torch.bfloat16)
    gates = _rnd(T, H, seed=3, dtype=torch.bfloat16)
    pos = torch.cat([torch.arange(c, c + n) for c, n in spans]).int()
    cs = ref.rope_cos_sin(800, rot_dims, 1000.0) if rot_dims else torch.zeros(800, 0, 2)
    wukv = _rnd(H * (dim + vdim), rank, seed=2, scale=rank ** -0.5).to(torch.bfloat16)
    k64 = -(-rank // 64) * 64
    dev = pack(step, 4, DEV)
    plan = long_spans(step, 256, window, ops.LATENT_ITEM, DEV)
    kd = kc.to(DEV)
    c = ops.latent_gather(kd, plan.pages, plan.valid, rank, torch.full(
        (plan.pages.numel() * 64, k64), 9.0, device=DEV, dtype=torch.bfloat16))
    assert torch.isfinite(c).all() and not c[:, rank:].any()
    w = torch.zeros(wukv.shape[0], k64, device=DEV, dtype=torch.bfloat16)
    w[:, :rank] = wukv
    out = torch.full((T, H, vdim), 5.0, device=DEV, dtype=torch.bfloat16)
    ops.latent_prefill(z, dev.attn, plan, pos.to(DEV), cs.to(DEV), H, dim, rot, ops.gemm(c, w), kd, rank, 0.05, window,
                       gates, out)
    qz = z[:, :H * (dim + rot)].float().cpu().view(T, H, dim + rot)
    q = torch.cat([qz[..., :dim], ref._rotate_halves(qz[..., dim:], cs[pos.long()])], -1)
    wk = wukv.float().cpu().view(H, dim + vdim, rank)
    for i, (ctx, n) in enumerate(spans):
        a = int(step.q_start[i])
        got = out[a:a + n].float().cpu()
        if n < 256:
            assert (got == 5).all()
            continue
        rows = torch.stack([kc[step.block_table[i, j // 64], 0, j % 64] for j in range(ctx + n)]).float()
        kv = torch.einsum("jr,hdr->hjd", rows[:, :rank], wk)
        mask = oracle.window_mask(ctx + n, window or ctx + n, 0)[ctx:]
        for h in range(H):
            s = (q[a:a + n, h, :dim] @ kv[h, :, :dim].T + q[a:a + n, h, dim:] @ rows[:, rank:rank + rot].T) * 0.05
            want = oracle.softmax(s, mask) @ kv[h, :, dim:] * torch.sigmoid(gates[a:a + n, h, None].float().cpu())
            _close(got[:, h], want, 2e-2)


def ops_row(rank, rot):
    """Cached row size of a latent layer."""
    return topelorn.LatentAttention(1, 32, rot, 64, rank, 0, 1.0, None).row[0]


# --------------------------------------------------------------------- model
TOL = {torch.float32: 4e-5, torch.bfloat16: 6e-2}
LENGTHS = (150, 65, 1, 320)


@pytest.fixture(scope="module")
def expected():
    """Oracle logits per configuration, computed once."""
    out = {}
    for name, c in cases.CONFIGS.items():
        w = cases.tensors(c, peaky=1.0)
        ps = cases.prompts(c, LENGTHS)
        out[name] = (c, w, ps, [cases.want_logits(c, w, p) for p in ps])
    return out


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", list(cases.CONFIGS))
def test_model_under_every_schedule(name, dtype, expected):
    c, w, ps, want = expected[name]
    model = cases.build(c, w, DEV, dtype)
    V = c["vocab"]
    for p, z in zip(ps, want):                              # whole; token by token; odd portions
        for sizes in ((len(p),), (1,), (63, 1, 2, 2, 64, 5, 30), (20, 300)):
            if sizes == (1,) and len(p) > 150:
                continue
            got = cases.replay(model, V, [[("a", t)] for t in cases.cuts(p, sizes)], 64 * (len(p) // 64 + 1))
            assert cases.error(got["a"], z) < TOL[dtype], (len(p), sizes)
    a, b, one, d = ps                                       # a mixed batch, requests of unequal length
    ca, cb, cd = cases.cuts(a, (37, 2, 1, 50)), cases.cuts(b, (10, 1)), cases.cuts(d, (270, 1, 3))
    steps = [[("b", cb[0])], [("d", cd[0]), ("b", cb[1])], [("a", ca[0]), ("d", cd[1]), ("x", one)]]
    rest = {"a": ca[1:], "b": cb[2:], "d": cd[2:]}
    while any(rest.values()):
        steps.append([(k, v.pop(0)) for k, v in rest.items() if v and (k != "b" or len(steps) % 3)])
        steps[-1] = steps[-1] or [("b", rest["b"].pop(0))]
    got = cases.replay(model, V, steps, 64 * 12)
    for k, z in (("a", want[0]), ("b", want[1]), ("x", want[2]), ("d", want[3])):
        assert cases.error(got[k], z) < TOL[dtype], k


def test_long_and_short_spans_share_a_step(expected):
    """Two long portions around short ones and single tokens in one batch."""
    c, w, ps, _ = expected["plain_sizes"]
    model = cases.build(c, w, DEV, torch.bfloat16)
    ps = cases.prompts(c, (700, 90, 40, 600), seed=9)
    want = [cases.want_logits(c, w, p) for p in ps]
    cd = cases.cuts(ps[3], (300,))
    steps = [[("b", ps[1][:60]), ("c", ps[2][:39])],
             [("d", cd[0]), ("c", ps[2][39:]), ("a", ps[0][:256]), ("b", ps[1][60:62])],
             [("b", ps[1][62:63]), ("a", ps[0][256:690]), ("d", cd[1])], [("a", ps[0][690:]), ("b", ps[1][63:])]]
    got = cases.replay(model, c["vocab"], steps, 64 * 26)
    for k, z in zip("abcd", want):
        assert cases.error(got[k], z) < TOL[torch.bfloat16], k


def test_a_long_span_equals_short_ones_up_to_rounding(expected):
    """Expanded and absorbed runs of the same prompt."""
    c, w, _, _ = expected["plain_sizes"]
    model = cases.build(c, w, DEV, torch.bfloat16)
    p = cases.prompts(c, (600,), seed=3)[0]
    z = cases.replay(model, c["vocab"], [[("a", p)]], 640)["a"]
    model.EXPAND_MIN = 10 ** 9
    y = cases.replay(model, c["vocab"], [[("a", p)]], 640)["a"]
    assert 0 < cases.error(y, z) < TOL[torch.bfloat16]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_pages_used_again(dtype, expected):
    """A pool that just holds two requests, many requests one after another in
    shifting pairs: freed pages come back with other requests' keys in them."""
    c, w, ps, want = expected["mixed"]
    model = cases.build(c, w, DEV, dtype)
    order = [0, 3, 1, 0, 3, 2, 3, 0, 1]
    steps, live = [], []
    for n, i in enumerate(order):
        parts = cases.cuts(ps[i], (80, 33, 1, 1, 40))
        live.append((f"r{n}", parts))
        if len(live) == 2:
            first, second = live
            while first[1]:
                steps.append([(first[0], first[1].pop(0))] + ([(second[0], second[1].pop(0))] if second[1] else []))
            live = [second] if second[1] else []
    for k, parts in live:
        steps += [[(k, t)] for t in parts]
    got = cases.replay(model, c["vocab"], steps, 64 * 9)
    for n, i in enumerate(order):
        assert cases.error(got[f"r{n}"], want[i]) < TOL[dtype], n


def test_layer_outputs():
    c = cases.CONFIGS["mixed"]
    w = cases.tensors(c)
    toks = cases.prompts(c, (90,))[0]
    layers = []
    oracle.forward(c, w, toks, layers_out=layers)
    model = cases.build(c, w, DEV, torch.float32)
    from mcp_amd.engine.batch import pack_step_py, to_device, views
    from mcp_amd.engine.kv_cache import KVCache
    host, layout = pack_step_py([(toks, 90, 0, [1, 0], 0, True)], BLOCK_SIZE, model.cfg.group)
    got = []
    model.forward(views(to_device(host, DEV), layout)[0], KVCache.for_model(model, 2),
                  tap=lambda r, x: got.append((r, x.clone())))
    assert [r for r, _ in got] == list(range(len(layers))) == list(range(6))
    for (r, x), want in zip(got, layers):
        _close(x.cpu(), want, 2e-5)


# -------------------------------------------------------------------- engine
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_greedy_generation_through_the_scheduler(dtype, expected):
    """generate(): graph replay and eager launches agree, and in 32 bits every
    token is the oracle's argmax (long enough to cross pages and windows)."""
    from mcp_amd.engine.engine import LLMEngine
    from mcp_amd.engine.generate import generate
    c, w, ps, _ = expected["mixed"]
    model = cases.build(c, w, DEV, dtype)
    prompts = [ps[0][:70], ps[1][:3], ps[2], ps[3][:125]]
    outs = []
    for graphs in (False, True):
        eng = LLMEngine(model, num_blocks=32, max_batch=8, temperature=0.0, graphs=graphs)
        outs.append(generate(eng, prompts, max_new=100))
        assert eng.alloc.num_free == eng.kv.num_blocks
        assert (eng.stats["graph_steps"] > 20) == graphs
    assert all(len(o) == 100 for o in outs[0])
    if dtype == torch.float32:
        assert outs[0] == outs[1]
        for p, o in zip(prompts, outs[0]):
            z = cases.want_logits(c, w, p + o)
            for i, t in enumerate(o):
                row = z[len(p) - 1 + i]
                assert row[t] >= row.max() - 1e-4 * np.abs(row).max(), i


def test_small_pool_preempts_and_recomputes(expected):
    from mcp_amd.engine.engine import LLMEngine
    from mcp_amd.engine.generate import generate
    c, w, ps, _ = expected["mixed"]
    model = cases.build(c, w, DEV, torch.float32)
    prompts = [ps[0][:60], ps[1][:50], ps[3][:62], ps[3][3:60], ps[0][5:60]]
    big = generate(LLMEngine(model, num_blocks=64, temperature=0.0, graphs=False), prompts, 40)
    eng = LLMEngine(model, num_blocks=7, temperature=0.0, graphs=False)
    assert generate(eng, prompts, 40) == big
    assert eng.stats["preemptions"] > 0


@pytest.mark.parametrize("name", ["plain_sizes", "wide_group"])
def test_graph_replays_match_eager_steps(name, expected):
    """One captured decode step replayed over several positions, other work in
    between, each replay against the eager step."""
    c, w, ps, want = expected[name]
    model = cases.build(c, w, DEV, torch.bfloat16)
    from mcp_amd.engine.batch import pack_step, to_device, views
    from mcp_amd.engine.kv_cache import KVCache
    kv = KVCache.for_model(model, 4)
    p = ps[3]

    def step(lo, hi, splits=1):
        host, layout = pack_step([(p[lo:hi], hi - lo, lo, [2, 0, 3, 1], 0, True)], BLOCK_SIZE, model.cfg.group)
        return torch.from_numpy(host), list(layout) + [splits, 0, 4]
    for splits in (1, 8):
        host, layout = step(0, 120)
        model.forward(views(host.to(DEV), layout)[0], kv)
        host, layout = step(120, 121, splits)
        buf = host.to(DEV)
        d = views(buf, layout)[0]
        model.forward(d, kv)
        torch.cuda.synchronize()
        g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g):
            out = model.forward(d, kv)
        for at in range(120, 140):
            buf.copy_(step(at, at + 1, splits)[0])
            g.replay()
            got = model.logits(out)
            torch.cuda.synchronize()
            eager = model.logits(model.forward(views(step(at, at + 1, splits)[0].to(DEV), layout)[0], kv))
            assert torch.equal(got, eager), at
            assert cases.error(got.float().cpu().numpy(), want[3][at:at + 1]) < TOL[torch.bfloat16]


def test_planner_serves_the_design():
    """Grammar-constrained planning on a random-init model of the registry."""
    from mcp_amd.engine.engine import LLMEngine
    from mcp_amd.models.registry import random_model
    from mcp_amd.orchestrator import validate_dag
    from mcp_amd.planner.local import LocalPlanner
    from mcp_amd.planner.prompt import synthetic_intent
    from mcp_amd.registry import MemoryRegistry, synthetic_registry
    model = random_model("topelorn-tiny", DEV, seed=2)
    reg = MemoryRegistry(synthetic_registry(8, seed=2))
    for graphs in (False, True):
        eng = LLMEngine(model, num_blocks=512, max_batch=32, temperature=0.0, graphs=graphs)
        outs = LocalPlanner(eng, reg, max_nodes=4, min_nodes=2).plan_many([synthetic_intent(i) for i in range(6)])
        assert eng.alloc.num_free == eng.kv.num_blocks and len(outs) == 6
        for d in outs:
            validate_dag(d, [s.name for s in reg.list_services()])


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_command(dtype, tmp_path, expected):
    from safetensors.torch import save_file
    c, w, ps, want = expected["mixed"]
    (tmp_path / "m").mkdir()
    (tmp_path / "o").mkdir()
    save_file(w, str(tmp_path / "m" / "model.safetensors"))
    (tmp_path / "m" / "config.json").write_text(json.dumps(copy.deepcopy(c)))
    a, b = ps[0], ps[1]
    steps = [{"entries": [{"id": "a", "tokens": a[:100], "want": [99, 0]}], "end": []},
             {"entries": [{"id": "b", "tokens": b, "want": []}, {"id": "a", "tokens": a[100:102], "want": [1]}],
              "end": ["b"]},
             {"entries": [{"id": "a", "tokens": a[102:103], "want": [0]}], "end": ["a"]}]
    # (the library is built already: the command's build step finds it up to date)
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", dtype,
                        "--out", str(tmp_path / "o"), "--max-tokens", "256"],
                       input="".join(json.dumps({"step": i, **s}) + "\n" for i, s in enumerate(steps)),
                       capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1", "done 2"]
    for i, at in ((0, [99, 0]), (1, [101]), (2, [102])):
        z = np.fromfile(tmp_path / "o" / f"{i}.f32", "<f4").reshape(len(at), c["vocab"])
        assert cases.error(z, want[0][at]) < TOL[getattr(torch, dtype)]
