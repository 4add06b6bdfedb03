"""Dozazen on the GPU: its kernels one by one against fp32 PyTorch, the model in
32 and 16 bits against the slow oracle under every way of cutting and batching,
generation through the scheduler, the trace command."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import mcp_amd.ops as ops
from mcp_amd.ops import reference as ref

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import dozazen_cases as cases  # noqa: E402
import dozazen_oracle as oracle  # noqa: E402

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
@pytest.mark.parametrize("rows,H,Hp", [(1, 100, 128), (3, 320, 320), (700, 200, 256), (1, 4096, 4096),
                                       (5, 5000, 5056), (600, 8192, 8192), (2, 16384, 16384)])
def test_residual_norm(rows, H, Hp, dtype):
    def padded(t):
        t[..., H:] = 0
        return t
    x, y = padded(_rnd(rows, Hp, seed=1)), padded(_rnd(rows, Hp, seed=2, scale=3.0)).to(dtype)
    wa, wb = padded(_rnd(Hp, seed=3)), padded(_rnd(Hp, seed=4))
    wide = torch.full((rows, 2 * Hp), 7.0, device=DEV, dtype=dtype)
    for kw in (dict(y=y, w_post=wa, w_pre=wb), dict(y=y, w_post=wa), dict(w_pre=wb), dict()):
        gx, wx = x.clone(), x.clone()
        got = ops.residual_norm(gx, H, 1e-5, out=wide[:, Hp:], **kw)
        want = ref.residual_norm(wx, H, 1e-5, out=torch.empty_like(y), **kw)
        _close(gx, wx, 1e-5)
        _close(got, want, 1e-5 if dtype == torch.float32 else 8e-3)
        assert (wide[:, :Hp] == 7).all()
    gx = x.clone()
    ops.residual_norm(gx, H, 1e-5, y, wa)                  # no output row wanted
    wx = x.clone()
    ref.residual_norm(wx, H, 1e-5, y, wa)
    _close(gx, wx, 1e-5)


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_embedding_scaled(dtype):
    table = _rnd(50, 320, dtype=dtype)
    ids = torch.tensor([3, 49, 0, 3], dtype=torch.int32, device=DEV)
    lo = torch.zeros(4, 640, device=DEV, dtype=dtype)
    x = ops.embedding_scaled(ids, table, 7.5, lo[:, 320:])
    want = table[ids.long()].float() * 7.5
    assert torch.equal(x, want) and torch.equal(lo[:, 320:], want.to(dtype)) and not lo[:, :320].any()


@pytest.mark.parametrize("M,N,K", [(1, 4, 64), (7, 100, 128), (65, 452, 320), (300, 260, 1024)])
def test_gemm_f32_is_exact_and_row_independent(M, N, K):
    X, W = _rnd(M, K, seed=1), _rnd(N, K, seed=2)
    got = ops.gemm(X, W)
    _close(got, X.double() @ W.double().t(), 2e-6)
    assert torch.equal(ops.gemm(X[-1:].contiguous(), W), got[-1:])


@pytest.mark.parametrize("M", [1, 3, 16, 40, 64, 100, 128, 200, 700, 2600])
@pytest.mark.parametrize("N,K", [(64, 128), (320, 640), (452, 320), (4096, 8192)])
def test_gemm_f32out(M, N, K):
    X, W = _rnd(M, K, seed=1, dtype=torch.bfloat16), _rnd(N, K, seed=2, dtype=torch.bfloat16)
    _close(ops.gemm_f32out(X, W), X.float() @ W.float().t(), 2e-5)


@pytest.mark.parametrize("M", [1, 4, 12, 33, 64, 100, 150, 200, 300, 520, 1100, 2600])
@pytest.mark.parametrize("F,K", [(64, 64), (192, 320), (14336, 4096)])
def test_gelu_gate_in_every_gemm_path(M, F, K):
    """The tanh form of gelu in the gated GEMM epilogue of every kernel the row
    count can pick; also that silu is what it was."""
    X = _rnd(M, K, seed=1, dtype=torch.bfloat16)
    W = ref.interleave_gate_up(_rnd(F, K, seed=2, scale=2 * K ** -0.5), _rnd(F, K, seed=3, scale=K ** -0.5))
    W = W.to(torch.bfloat16)
    y = X.float() @ W.float().t()
    y = y.view(M, F // 16, 2, 16)
    g, u = y[:, :, 0].reshape(M, F), y[:, :, 1].reshape(M, F)
    _close(ops.gemm_silu(X, W, act="gelu_tanh"), torch.nn.functional.gelu(g, approximate="tanh") * u, 6e-3)
    _close(ops.gemm_silu(X, W), torch.nn.functional.silu(g) * u, 6e-3)


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("M", [1, 20, 60, 100, 130, 300, 700, 2600])
@pytest.mark.parametrize("Hq,Hkv,DK,DV,K", [(6, 3, 64, 64, 320), (6, 2, 128, 64, 64), (4, 2, 128, 128, 256),
                                            (32, 8, 128, 128, 4096)])
def test_qkv_rope_bias(M, Hq, Hkv, DK, DV, K, dtype):
    if dtype == torch.float32 and K == 4096 and M > 300:
        pytest.skip("32-bit mode: small sizes are enough")
    N = (Hq + Hkv) * DK + Hkv * DV
    h, W = _rnd(M, K, seed=1, dtype=dtype), _rnd(N, K, seed=2, dtype=dtype, scale=K ** -0.5)
    bias = _rnd(N, seed=3)
    pos = torch.randint(0, 500, (M,), generator=torch.Generator().manual_seed(4)).int()
    nb = M // 64 + 2
    slots = torch.randperm(nb * 64, generator=torch.Generator().manual_seed(5))[:M].int()
    slots[M // 2] = -1 if M > 1 else slots[0]
    cs = torch.randn(500, DK // 2, 2, generator=torch.Generator().manual_seed(6))

    def run(f, dev, dt):
        q = torch.zeros(M, Hq, DK, device=dev, dtype=dt)
        kc = torch.zeros(nb, Hkv, 64, DK, device=dev, dtype=dt)
        vc = torch.zeros(nb, Hkv, 64, DV, device=dev, dtype=dt)
        f(q, kc, vc, pos.to(dev), slots.to(dev), cs.to(dev))
        return q, kc, vc
    got = run(lambda q, kc, vc, p, s, c: ops.qkv_rope_bias(h, W, bias, p, s, c, q, kc, vc), DEV, dtype)
    z = (h.float() @ W.float().t() + bias).cpu()
    want = run(lambda q, kc, vc, p, s, c: ref.rope_kv_any(z, p, s, c, q, kc, vc), "cpu", torch.float32)
    for g, w in zip(got, want):
        _close(g.cpu().float(), w, 1.6e-2 if dtype == torch.bfloat16 else 1e-5)


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_sampling_scales_and_caps_logits(dtype):
    R, V, H = 5, 300, 128
    hid, W = _rnd(R, H, seed=1, dtype=dtype), _rnd(V, H, seed=2, dtype=dtype)
    z = ref.soft_cap(hid.double() @ W.double().t() * 0.5, 3.0)
    ptr = torch.tensor([0, 3, 3, 4, 9, 10], dtype=torch.int32, device=DEV)
    ids = torch.tensor([5, 17, 299, -1, 4, 9, 2, 200, 100, 44], dtype=torch.int32, device=DEV)
    ctr = torch.arange(R, dtype=torch.int32, device=DEV)
    logits = ops.logit_finish(ops.gemm_f32out(hid, W), 0.5, 3.0)
    _close(logits, z, 2e-5)
    tok = ops.sample_dense(logits, ptr, ids, ctr, 0.0, 0).tolist()
    sets = [ids[ptr[i]:ptr[i + 1]].tolist() for i in range(R)]
    want = [-1 if not s else (int(z[i].argmax()) if s == [-1] else max(s, key=lambda t: float(z[i, t])))
            for i, s in enumerate(sets)]
    assert tok == want
    # the fused head: logits of the allowed rows, scaled and capped
    sets = [[5, 17, 299], [8], [1], [4, 9, 2, 200], [100]]
    ptr2 = torch.tensor(np.cumsum([0] + [len(s) for s in sets]), dtype=torch.int32, device=DEV)
    ids2 = torch.tensor(sum(sets, []), dtype=torch.int32, device=DEV)
    out_logit = torch.empty(R, device=DEV)
    tok = ops.sample_allowed(hid, W, ptr2, ids2, ctr, 0.0, 0, out_logit=out_logit, logit_scale=0.5,
                             logit_cap=3.0).tolist()
    assert tok == [max(s, key=lambda t: float(z[i, t])) for i, s in enumerate(sets)]
    _close(out_logit, z[torch.arange(R), torch.tensor(tok)], 2e-5)
    # sampling follows the capped distribution
    n = 20000
    two = logits[:1, :2].contiguous().expand(n, 2).contiguous()
    t = ops.sample_dense(two, torch.arange(n + 1, dtype=torch.int32, device=DEV),
                         torch.full((n,), -1, dtype=torch.int32, device=DEV),
                         torch.arange(n, dtype=torch.int32, device=DEV), 1.0, 3)
    p = float(torch.softmax(z[0, :2], 0)[1])
    assert abs(float(t.float().mean()) - p) < 0.02


def test_cache_of_unequal_layers_copies_blocks():
    from mcp_amd.engine.kv_cache import KVCache
    for dtype in (torch.bfloat16, torch.float32):
        kv = KVCache.from_specs([(2, 64, 128), (1, 64, 64), (2, 64, 128)], 6, DEV, dtype)
        for t in kv.stacks:
            t.normal_()
        before = [[t.clone() for t in kv.layer(i)] for i in range(3)]
        kv.copy_blocks(torch.tensor([1, -1, 4], dtype=torch.int32, device=DEV),
                       torch.tensor([3, -1, 0], dtype=torch.int32, device=DEV))
        for i in range(3):
            for t, b in zip(kv.layer(i), before[i]):
                assert torch.equal(t[3], b[1]) and torch.equal(t[0], b[4])
                assert torch.equal(t[[1, 2, 4, 5]], b[[1, 2, 4, 5]])


# --------------------------------------------------------------------- model
TOL = {torch.float32: 2e-5, torch.bfloat16: 6e-2}
LENGTHS = (150, 65, 1, 203)


@pytest.fixture(scope="module")
def expected():
    """Oracle logits per configuration, computed once."""
    out = {}
    for name, c in cases.CONFIGS.items():
        w = cases.tensors(c)
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
        for sizes in ((len(p),), (1,), (63, 1, 2, 2, 64, 5, 30)):
            if sizes == (1,) and len(p) > 150:
                continue
            got = cases.replay(model, V, [[("a", t)] for t in cases.cuts(p, sizes)], 64 * (len(p) // 64 + 1))
            assert cases.error(got["a"], z) < TOL[dtype], (len(p), sizes)
    a, b, one, d = ps                                       # a mixed batch, requests of unequal length
    ca, cb, cd = cases.cuts(a, (37, 2, 1, 50)), cases.cuts(b, (10, 1)), cases.cuts(d, (128, 1, 3))
    steps = [[("d", cd[0]), ("b", cb[0])], [("a", ca[0]), ("d", cd[1]), ("x", one)]]
    rest = {"a": ca[1:], "b": cb[1:], "d": cd[2:]}
    while any(rest.values()):
        steps.append([(k, v.pop(0)) for k, v in rest.items() if v and (k != "b" or len(steps) % 3)])
        steps[-1] = steps[-1] or [("b", rest["b"].pop(0))]
    got = cases.replay(model, V, steps, 64 * 10)
    for k, z in (("a", want[0]), ("b", want[1]), ("x", want[2]), ("d", want[3])):
        assert cases.error(got[k], z) < TOL[dtype], k


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
    got = cases.replay(model, c["vocab"], steps, 64 * 7)
    for n, i in enumerate(order):
        assert cases.error(got[f"r{n}"], want[i]) < TOL[dtype], n


def test_chunk_edges_in_the_model():
    """Far keys that stand out: the same token again just inside and just
    outside the chunk, prompts and decoding, against the oracle."""
    c = json.loads(json.dumps(cases.CONFIGS["no_loop"]))
    w = cases.tensors(c, seed=5, peaky=8.0)
    model = cases.build(c, w, DEV, torch.float32)
    size = c["layers"][0]["mixer"]["mask"]["size"]
    for n in (size - 1, size, size + 1, 2 * size, 2 * size + 1, 3 * size + 14):
        p = cases.prompts(c, (n + 1,), seed=n)[0]
        p[n // size * size] = p[n]
        if n // size:
            p[n // size * size - 1] = p[n]
        z = cases.want_logits(c, w, p)
        for sizes in ((len(p),), (n, 1), (size, 1), (size - 1, 2, 2)):
            got = cases.replay(model, c["vocab"], [[("a", t)] for t in cases.cuts(p, sizes)], 64 * 4)
            assert cases.error(got["a"], z) < TOL[torch.float32], (n, sizes)


def test_layer_outputs():
    c = cases.CONFIGS["mixed"]
    w = cases.tensors(c)
    toks = cases.prompts(c, (90,))[0]
    layers = []
    oracle.forward(c, w, toks, layers_out=layers)
    model = cases.build(c, w, DEV, torch.float32)
    from mcp_amd.engine.batch import BLOCK_SIZE, pack_step_py, to_device, views
    from mcp_amd.engine.kv_cache import KVCache
    host, layout = pack_step_py([(toks, 90, 0, [1, 0], 0, True)], BLOCK_SIZE, model.cfg.group)
    got = []
    model.forward(views(to_device(host, DEV), layout)[0], KVCache.for_model(model, 2),
                  tap=lambda r, x: got.append((r, x.clone())))
    assert [r for r, _ in got] == list(range(len(layers))) == list(range(8))
    for (r, x), want in zip(got, layers):
        _close(x.cpu(), want, 2e-5)


# -------------------------------------------------------------------- engine
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_greedy_generation_through_the_scheduler(dtype, expected):
    """generate(): graph replay and eager launches agree, and in 32 bits every
    token is the oracle's argmax (long enough to cross pages and chunks)."""
    from mcp_amd.engine.engine import LLMEngine
    from mcp_amd.engine.generate import generate
    c, w, ps, _ = expected["mixed"]
    model = cases.build(c, w, DEV, dtype)
    prompts = [ps[0][:70], ps[1][:3], ps[2], ps[3][:125]]
    outs = []
    for graphs in (False, True):
        eng = LLMEngine(model, num_blocks=32, max_batch=8, temperature=0.0, graphs=graphs)
        outs.append(generate(eng, prompts, max_new=48))
        assert eng.alloc.num_free == eng.kv.num_blocks
        assert (eng.stats["graph_steps"] > 20) == graphs
    assert outs[0] == outs[1] and all(len(o) == 48 for o in outs[0])
    if dtype == torch.float32:
        for p, o in zip(prompts, outs[0]):
            z = cases.want_logits(c, w, p + o)
            for i, t in enumerate(o):
                row = z[len(p) - 1 + i]
                assert row[t] >= row.max() - 1e-4 * np.abs(row).max(), i


def test_small_pool_preempts_and_recomputes(expected):
    """More requests than the pool holds: admission waits, requests are
    preempted and recomputed, the tokens stay those of an ample pool."""
    from mcp_amd.engine.engine import LLMEngine
    from mcp_amd.engine.generate import generate
    c, w, ps, _ = expected["mixed"]
    model = cases.build(c, w, DEV, torch.float32)
    prompts = [ps[0][:60], ps[1][:50], ps[3][:62], ps[3][3:60], ps[0][5:60]]
    big = generate(LLMEngine(model, num_blocks=64, temperature=0.0, graphs=False), prompts, 40)
    eng = LLMEngine(model, num_blocks=7, temperature=0.0, graphs=False)
    assert generate(eng, prompts, 40) == big
    assert eng.stats["preemptions"] > 0


def test_graph_replays_match_eager_steps(expected):
    """One captured decode step replayed over several positions, other work in
    between, each replay against the eager step."""
    c, w, ps, want = expected["whole_loop"]
    model = cases.build(c, w, DEV, torch.bfloat16)
    from mcp_amd.engine.batch import BLOCK_SIZE, pack_step, to_device, views
    from mcp_amd.engine.kv_cache import KVCache
    kv = KVCache.for_model(model, 4)
    p = ps[3]

    def step(lo, hi, splits=1):
        host, layout = pack_step([(p[lo:hi], hi - lo, lo, [2, 0, 3, 1], 0, True)], BLOCK_SIZE, model.cfg.group)
        return torch.from_numpy(host), list(layout) + [splits, 0, 4]
    for splits in (1, 8):
        host, layout = step(0, 60)
        model.forward(views(host.to(DEV), layout)[0], kv)
        host, layout = step(60, 61, splits)
        buf = host.to(DEV)
        d = views(buf, layout)[0]
        model.forward(d, kv)
        torch.cuda.synchronize()
        g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g):
            out = model.forward(d, kv)
        for at in range(60, 72):
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
    model = random_model("dozazen-tiny", DEV, seed=2)
    reg = MemoryRegistry(synthetic_registry(8, seed=2))
    outs = []
    for graphs in (False, True):
        eng = LLMEngine(model, num_blocks=512, max_batch=32, temperature=0.0, graphs=graphs)
        outs.append(LocalPlanner(eng, reg, max_nodes=4, min_nodes=2).plan_many(
            [synthetic_intent(i) for i in range(6)]))
        assert eng.alloc.num_free == eng.kv.num_blocks
    assert outs[0] == outs[1]
    for d in outs[0]:
        validate_dag(d, [s.name for s in reg.list_services()])


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_command(dtype, tmp_path, expected):
    from safetensors.torch import save_file
    c, w, ps, want = expected["whole_loop"]
    (tmp_path / "m").mkdir()
    (tmp_path / "o").mkdir()
    save_file(w, str(tmp_path / "m" / "model.safetensors"))
    (tmp_path / "m" / "config.json").write_text(json.dumps(c))
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
