"""Masked paged attention (csrc/attention_masked.hip) against fp32 PyTorch: soft
cap, chunked mask, sink, unequal key / value heads, any GQA group, ragged
batches over shuffled pages with stale contents, split keys."""
import numpy as np
import pytest
import torch

import mcp_amd.ops as ops
from mcp_amd.engine.batch import StepInputs, pack
from mcp_amd.models.llama import padded_group
from mcp_amd.ops import reference as ref

pytestmark = pytest.mark.gpu
DEV = "cuda"
BS = 64


def _case(spans, Hq, Hkv, DK, DV, dtype, seed=0, stale=True, amp=1.0):
    """spans: (context before, new tokens) per sequence, pages shuffled."""
    g = torch.Generator().manual_seed(seed)
    need = [(c + n + BS - 1) // BS for c, n in spans]
    nb = sum(need) + 3
    perm = torch.randperm(nb, generator=g).tolist()
    kc = torch.randn(nb, Hkv, BS, DK, generator=g) * amp
    vc = torch.randn(nb, Hkv, BS, DV, generator=g)
    T = sum(n for _, n in spans)
    q = torch.randn(T, Hq, DK, generator=g) * amp
    bt = np.zeros((len(spans), max(need)), np.int32)
    qs, at = [], 0
    for i, (c, n) in enumerate(spans):
        bt[i, :need[i]] = [perm.pop() for _ in range(need[i])]
        qs.append(at)
        at += n
        if stale:      # places past the last key hold whatever an earlier request left
            b, o = bt[i, (c + n - 1) // BS], (c + n - 1) % BS + 1
            kc[b, :, o:] = float("nan")
            vc[b, :, o:] = float("nan")
    step = StepInputs(token_ids=np.zeros(T, np.int32), positions=np.zeros(T, np.int32),
                      slots=np.zeros(T, np.int32), q_start=np.asarray(qs, np.int32),
                      q_len=np.asarray([n for _, n in spans], np.int32),
                      ctx_len=np.asarray([c + n for c, n in spans], np.int32), block_table=bt,
                      logit_rows=np.zeros(0, np.int32))
    return q.to(dtype), kc.to(dtype), vc.to(dtype), step


def _check(spans, Hq, Hkv, DK, DV, cap, chunk, sink, dtype=torch.bfloat16, splits=1, seed=0, amp=1.0):
    q, kc, vc, step = _case(spans, Hq, Hkv, DK, DV, dtype, seed, amp=amp)
    group = padded_group(min(Hq // Hkv, 16))
    dev = pack(step, group, DEV)
    dev.attn.kv_splits = splits
    scale = DK ** -0.5
    got = ops.masked_attention(q.to(DEV), kc.to(DEV), vc.to(DEV), dev.attn, scale, group, cap, chunk, sink)
    t = lambda a: torch.from_numpy(np.asarray(a))
    want = ref.masked_attention(q.float(), kc.float().nan_to_num(), vc.float().nan_to_num(), t(step.q_start),
                                t(step.q_len), t(step.ctx_len), t(step.block_table), scale, cap, chunk, sink)
    d = (got.float().cpu() - want)
    assert torch.isfinite(got).all()
    tol = 2e-5 if dtype == torch.float32 else 1.2e-2
    err = d.abs().amax(dim=(1, 2)) / want.abs().amax()
    assert err.max() < tol, (float(err.max()), int(err.argmax()))


MIXED = [(0, 70), (63, 1), (64, 1), (190, 3), (0, 1), (129, 40), (255, 2)]


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("Hq,Hkv,DK,DV", [(6, 2, 64, 64), (8, 2, 128, 128), (6, 2, 128, 64), (5, 5, 64, 128),
                                          (40, 2, 64, 64), (7, 1, 192, 128), (4, 2, 256, 256), (4, 4, 64, 192)])
def test_head_shapes(Hq, Hkv, DK, DV, dtype):
    _check(MIXED, Hq, Hkv, DK, DV, 30.0, 50, True, dtype)


@pytest.mark.parametrize("cap", [0.0, 2.0, 50.0, 200.0])
@pytest.mark.parametrize("chunk", [0, 1, 7, 64, 100, 128, 5000])
@pytest.mark.parametrize("sink", [False, True])
def test_masks_caps_sinks(cap, chunk, sink):
    _check(MIXED, 8, 2, 128, 128, cap, chunk, sink, amp=2.0, seed=chunk)


@pytest.mark.parametrize("splits", [2, 4, 8, 32])
@pytest.mark.parametrize("cap", [0.0, 50.0, 100.0])
def test_split_keys(splits, cap):
    _check([(1500, 1), (70, 1), (0, 2), (999, 3), (640, 1)], 8, 2, 128, 128, cap, 700, True, splits=splits)
    _check([(1500, 1), (63, 1)], 6, 2, 64, 128, cap, 0, False, splits=splits)


@pytest.mark.parametrize("chunk", [100, 128, 192])
def test_chunk_edges_stand_out(chunk):
    """One huge key just inside and one just outside the chunk: a mask that is
    one position off changes the output completely."""
    for pos in (chunk - 1, chunk, chunk + 1, 2 * chunk - 1, 2 * chunk, 2 * chunk + 63):
        for new in (1, 2, 5, pos + 1):
            if new > pos + 1:
                continue
            q, kc, vc, step = _case([(pos + 1 - new, new)], 2, 1, 64, 64, torch.bfloat16, seed=pos)
            first = pos // chunk * chunk
            bt = step.block_table[0]
            u = torch.randn(64, generator=torch.Generator().manual_seed(pos))
            u = (u / u.norm() * 16).to(torch.bfloat16)
            q[-1] = u
            for key, v in ((first, 3.0), (first - 1, -50.0)):
                if key >= 0:
                    kc[bt[key // BS], 0, key % BS] = u
                    vc[bt[key // BS], 0, key % BS] = v
            dev = pack(step, 4, DEV)
            got = ops.masked_attention(q.to(DEV), kc.to(DEV), vc.to(DEV), dev.attn, 64 ** -0.5, 4, 30.0,
                                       chunk, True)[-1].float()
            assert (got - 3.0).abs().max() < 0.05, (pos, new, got.flatten()[:4])


def test_sink_without_keys_in_reach_of_zero():
    """Scores far below the sink's 0: the sink takes nearly all the weight."""
    q, kc, vc, step = _case([(30, 2)], 2, 1, 64, 64, torch.bfloat16)
    q[:] = 1.0
    kc[:] = torch.where(kc.isnan(), kc, torch.full_like(kc, -1.0))     # score -8 before the cap
    vc[:] = torch.where(vc.isnan(), vc, torch.ones_like(vc))
    dev = pack(step, 4, DEV)
    got = ops.masked_attention(q.to(DEV), kc.to(DEV), vc.to(DEV), dev.attn, 0.125, 4, 50.0, 0, True).float().cpu()
    s = 50 * np.tanh(-8 / 50)
    for i, n in enumerate((31, 32)):
        w = n * np.exp(s) / (1 + n * np.exp(s))
        assert abs(float(got[i, 0, 0]) - w) < 0.01 * w


def test_rows_do_not_depend_on_the_batch_or_pages():
    spans = [(130, 1), (0, 90), (77, 5)]
    q, kc, vc, step = _case(spans, 8, 2, 128, 128, torch.bfloat16, seed=3)
    k = dict(soft_cap=30.0, chunk=100, sink=True)
    dev = pack(step, 4, DEV)
    alls = ops.masked_attention(q.to(DEV), kc.to(DEV), vc.to(DEV), dev.attn, 0.09, 4, **k)
    for i, (c, n) in enumerate(spans):
        a = int(step.q_start[i])
        one = StepInputs(np.zeros(n, np.int32), np.zeros(n, np.int32), np.zeros(n, np.int32),
                         np.zeros(1, np.int32), step.q_len[i:i + 1], step.ctx_len[i:i + 1],
                         step.block_table[i:i + 1], np.zeros(0, np.int32))
        alone = ops.masked_attention(q[a:a + n].to(DEV).contiguous(), kc.to(DEV), vc.to(DEV),
                                     pack(one, 4, DEV).attn, 0.09, 4, **k)
        assert torch.equal(alone, alls[a:a + n])
