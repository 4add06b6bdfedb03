"""Prefill and decode throughput of one design's layers beside another's.

``bench.py --compare dozazen`` (or ``topelorn``) runs it: a few decoder layers with the sizes of a
real model, random weights, on the engine's own step descriptors and paged cache
- a prompt step eagerly, decode steps as the replayed hipGraph they are when
served - for the design and for Llama at equal sizes, the two alternating.  One
JSON line per (sizes, phase).
"""
from __future__ import annotations

import dataclasses
import json
import statistics
import time

import numpy as np
import torch

LAYERS = 4
VOCAB = 32768
# name: (width, heads, kv_heads, head_dim, ffn)
SIZES = {"1b": (2048, 16, 4, 128, 8192), "8b": (4096, 32, 8, 128, 14336), "70b": (8192, 64, 8, 128, 28672)}
# name: (sequences, context before the step, new tokens per sequence)
PHASES = {"prefill_1x4096": (1, 0, 4096), "prefill_4x1024": (4, 0, 1024), "decode_1_ctx2048": (1, 2047, 1),
          "decode_16_ctx2048": (16, 2047, 1), "decode_64_ctx1024": (64, 1023, 1)}


def _models(size: str, device, which):
    from ..models import dozazen, llama, topelorn
    W, H, G, D, F = SIZES[size]
    out = {}
    if "llama" in which:
        cfg = dataclasses.replace(llama.CONFIGS["llama3-8b"], name=f"llama-{size}", layers=LAYERS, hidden=W,
                                  heads=H, kv_heads=G, head_dim=D, ffn=F, vocab_size=VOCAB)
        out["llama"] = llama.LlamaModel(cfg, llama.random_weights(cfg, device, seed=1), device)
    if "dozazen" in which:
        # equal layer runs: one layer twice, the others once
        cfg = dozazen.uniform_config(f"dozazen-{size}", LAYERS - 1, W, H, G, D, F, VOCAB, 8192,
                                     loop=(1, 2, 2), max_pos=8192)
        out["dozazen"] = dozazen.DozazenModel.random(cfg, device, seed=1)
    if "topelorn" in which:
        # attention and latent layers in turn, windows no shorter than Llama's spans here
        cfg = topelorn.alternating_config(f"topelorn-{size}", LAYERS, W, H, G, D, F, VOCAB, max_pos=8192)
        out["topelorn"] = topelorn.TopelornModel.random(cfg, device, seed=1)
    return out


def _step(model, seqs: int, ctx: int, new: int, device):
    from ..engine.batch import BLOCK_SIZE, choose_kv_splits, pack_step, step_from_host, to_device, views
    from ..engine.kv_cache import KVCache
    need = -(-(ctx + new) // BLOCK_SIZE)
    kv = KVCache.for_model(model, seqs * need)
    for t in kv.stacks:
        t.normal_(0, 0.5)
    perm = np.random.default_rng(0).permutation(seqs * need).tolist()
    toks = np.random.default_rng(1).integers(0, VOCAB, new).tolist()
    entries = [(toks, new, ctx, perm[i * need:(i + 1) * need], 0, True) for i in range(seqs)]
    host, layout = pack_step(entries, BLOCK_SIZE, model.cfg.group)
    own = [ctx + new] * seqs
    ns = choose_kv_splits([new] * seqs, own, model.cfg.group, model.hkv, hq=model.hq)
    d = views(to_device(host, device), list(layout) + [ns, 0, -(-(ctx + new) // BLOCK_SIZE)])[0]
    if getattr(model, "uses_host_step", False) and new > 1:
        d.attn.host = step_from_host(host, layout)
    return d, kv


def _runner(model, phase: str, device):
    seqs, ctx, new = PHASES[phase]
    d, kv = _step(model, seqs, ctx, new, device)
    model.forward(d, kv)
    torch.cuda.synchronize()
    if not phase.startswith("decode"):
        return lambda: model.forward(d, kv), (d, kv)
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        out = model.forward(d, kv)
    return g.replay, (d, kv, g, out)


def _time(fn, reps: int) -> float:
    torch.cuda.synchronize()
    t = time.perf_counter()
    for _ in range(reps):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t) / reps


def run(design: str = "dozazen", sizes=None, phases=None, which=None, device="cuda:0", log=print):
    which = which or ("llama", design)
    for size in sizes or SIZES:
        models = _models(size, device, which)
        for phase in phases or PHASES:
            seqs, ctx, new = PHASES[phase]
            fns = {n: _runner(m, phase, device) for n, m in models.items()}
            for fn, _ in fns.values():
                _time(fn, 3)
            t0 = time.perf_counter()
            ms = {n: [] for n in fns}
            reps = 5 if phase.startswith("prefill") else 50
            while min(len(v) for v in ms.values()) < 7 and time.perf_counter() - t0 < 10:
                for n, (fn, _) in fns.items():
                    ms[n].append(_time(fn, reps) * 1e3)
            line = {"layers": LAYERS, "size": size, "phase": phase}
            for n, v in ms.items():
                med = statistics.median(v)
                line[n] = {"ms": round(med, 4), "tokens_per_s": round(seqs * new / med * 1e3, 1)}
            if len(ms) == 2:
                a, b = (statistics.median(v) for v in ms.values())
                line["time_ratio"] = round(b / a, 3)
            log(json.dumps(line), flush=True)
            del fns
        del models
        torch.cuda.empty_cache()
