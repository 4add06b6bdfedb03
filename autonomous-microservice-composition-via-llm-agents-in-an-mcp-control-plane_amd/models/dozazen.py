"""Dozazen decoder: chunked attention with capped scores and a softmax sink,
norms on both sides of every sublayer, a run of layers repeated with the same
weights, an fp32 residual stream.

One ragged, paged step (n = rms norm with its own weight, c(z; k) = k tanh(z / k)):

    x0 = x = embed(ids) * embed_scale                     fp32 residual
    per layer run:
        at the start of a pass of the repeated layers:  x = [x ; x0] W_loop^T
        q, k, v = n1(x) Wqkv^T + b;  q, k rotated         K/V into the run's own cache layer
        s = c(q k * scale; cap) over the keys of the query's own chunk
        a = sum_j e^{s_j} v_j / (1 + sum_j e^{s_j})
        x = x + n1b(a Wo^T)
        x = x + n2b((gelu(n2(x) Wg^T) * (n2(x) Wu^T)) Wd^T)    layers with a feed-forward
    logits = c(n(x) head^T * logit_scale; logit_cap)

What this module adds to the shared machinery is the mapping onto it:

* every size is padded to what the MFMA kernels tile by (width and feed-forward
  to 64, head sizes to ``ops.HEAD_SIZES``) with zero rows / columns, which is exact;
* neighbouring-pair rotation becomes the kernels' half rotation by permuting the
  rows of Wq / Wk (the same permutation on both leaves q . k unchanged); pairs
  that do not rotate (partial rotation, padding) hold (1, 0) in the table;
* between two sublayers ONE pass over the residual does post-norm, add and the
  next pre-norm (``ops.residual_norm``), so the projections see normed rows;
* each run of a repeated layer is a cached layer of its own (``kv_specs``).

``dtype`` float32 weights run everything in 32 bits, the caches included.
"""
from __future__ import annotations

import dataclasses
import json
from pathlib import Path
from typing import Dict, List, Optional, Tuple

import torch

from .. import ops
from ..ops import reference as ref
from .llama import padded_group
from .packing import MAX_POS, Rotary, head_size, rope_table
from .packing import leading as _leading, pad as _pad, pick_rows as _pick_rows, up as _up


@dataclasses.dataclass(frozen=True)
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int                  # query / key head size
    vdim: int                 # value head size
    chunk: int                # tokens per attention chunk (0: one chunk)
    rot: Rotary
    scale: float
    soft_cap: float = 0.0


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: AttentionSpec
    ffn: Optional[int]        # feed-forward width, None: no feed-forward


@dataclasses.dataclass(frozen=True)
class DozazenConfig:
    name: str
    vocab_size: int
    width: int
    layer_specs: Tuple[LayerSpec, ...]
    loop: Optional[Tuple[int, int, int]] = None      # layers [start, stop) run ``times`` times
    embed_scale: float = 1.0
    logit_scale: float = 1.0
    logit_cap: float = 0.0
    eps: float = 1e-5
    max_pos: int = MAX_POS

    def runs(self) -> List[Tuple[int, bool]]:
        """(layer, begins a pass of the repeated layers) in execution order."""
        n = len(self.layer_specs)
        if self.loop is None:
            return [(i, False) for i in range(n)]
        start, stop, times = self.loop
        return ([(i, False) for i in range(start)]
                + [(i, i == start) for _ in range(times) for i in range(start, stop)]
                + [(i, False) for i in range(stop, n)])

    @property
    def layers(self) -> int:
        """Cached layers: one per layer run."""
        return len(self.runs())

    @property
    def hidden(self) -> int:
        return self.width

    @property
    def group(self) -> int:
        """Query heads per key head the attention work items are cut for (the
        kernels take any group; larger ones walk several row tiles)."""
        g = max(s.mixer.heads // s.mixer.kv_heads for s in self.layer_specs)
        return padded_group(min(g, 16))

    def params(self) -> int:
        W, n = self.width, 2 * self.vocab_size * self.width + self.width
        for s in self.layer_specs:
            m = s.mixer
            n += (W + 1) * (m.heads * m.dim + m.kv_heads * (m.dim + m.vdim)) + W * m.heads * m.vdim
            n += 2 * W + (0 if s.ffn is None else 3 * W * s.ffn + 2 * W)
        return n + (2 * W * W if self.loop else 0)


def config_from_json(c: dict, name: str = "dozazen", max_pos: int = MAX_POS) -> DozazenConfig:
    specs = []
    for i, ly in enumerate(c["layers"]):
        if ly["type"] != "attention":
            raise NotImplementedError(f"layer {i}: mixer type {ly['type']!r}")
        m, mlp = ly["mixer"], ly.get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise NotImplementedError(f"layer {i}: feed-forward kind {mlp['kind']!r}")
        r = m.get("rot") or {"dims": 0, "base": 1.0}
        sc = r.get("scaling")
        if m["heads"] % m["kv_heads"] or r["dims"] % 2 or r["dims"] > m["dim"]:
            raise ValueError(f"layer {i}: heads {m['heads']} / {m['kv_heads']}, rotated dimensions "
                             f"{r['dims']} of {m['dim']}")
        rot = Rotary(int(r["dims"]), float(r["base"]),
                     None if not sc else (float(sc["factor"]), float(sc["low"]), float(sc["high"]),
                                          float(sc["original"])))
        specs.append(LayerSpec(
            AttentionSpec(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]),
                          int((m.get("mask") or {}).get("size") or 0), rot, float(m["scale"]),
                          float(m.get("softcap") or 0.0)),
            None if mlp is None else int(mlp["ff"])))
    lp = c.get("loop")
    if lp and not 0 <= lp["start"] < lp["stop"] <= len(specs):
        raise ValueError(f"loop over layers {lp['start']} .. {lp['stop'] - 1} of {len(specs)}")
    return DozazenConfig(
        name=name, vocab_size=int(c["vocab"]), width=int(c["width"]), layer_specs=tuple(specs),
        loop=(int(lp["start"]), int(lp["stop"]), int(lp["times"])) if lp else None,
        embed_scale=float(c["embedding"]["scale"]), logit_scale=float(c.get("logit_scale") or 1.0),
        logit_cap=float(c.get("logit_softcap") or 0.0), eps=float(c["norm"]["eps"]), max_pos=max_pos)


def config_to_json(cfg: DozazenConfig) -> dict:
    layers = []
    for s in cfg.layer_specs:
        m = s.mixer
        sc = m.rot.scaling
        layers.append({"type": "attention", "mlp": None if s.ffn is None else {"kind": "dense", "ff": s.ffn},
                       "mixer": {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim,
                                 "mask": {"size": m.chunk}, "scale": m.scale, "softcap": m.soft_cap,
                                 "rot": {"dims": m.rot.dims, "base": m.rot.base, "scaling": None if sc is None
                                         else dict(zip(("factor", "low", "high", "original"), sc))}}})
    return {"architecture": "Dozazen", "vocab": cfg.vocab_size, "width": cfg.width, "layers": layers,
            "loop": dict(zip(("start", "stop", "times"), cfg.loop)) if cfg.loop else None,
            "embedding": {"scale": cfg.embed_scale}, "norm": {"eps": cfg.eps},
            "logit_scale": cfg.logit_scale, "logit_softcap": cfg.logit_cap}


def uniform_config(name: str, layers: int, width: int, heads: int, kv_heads: int, dim: int, ffn: int,
                   vocab_size: int, chunk: int, loop=None, vdim: Optional[int] = None,
                   **kw) -> DozazenConfig:
    """Equal layers (benchmarks, tests, named random-init models)."""
    m = AttentionSpec(heads, kv_heads, dim, vdim or dim, chunk,
                      Rotary(dim, 500000.0, (8.0, 1.0, 4.0, 8192.0)), dim ** -0.5, 50.0)
    kw = {"logit_cap": 30.0, **kw}
    return DozazenConfig(name, vocab_size, width, (LayerSpec(m, ffn),) * layers, loop=loop, **kw)


CONFIGS: Dict[str, DozazenConfig] = {
    # the layer sizes of an 8B model, 32 layer runs: 22 layers' weights, the 10
    # middle ones run twice
    "dozazen-8b": uniform_config("dozazen-8b", 22, 4096, 32, 8, 128, 14336, 128256, 8192, (6, 16, 2)),
    "dozazen-8b-2l": uniform_config("dozazen-8b-2l", 2, 4096, 32, 8, 128, 14336, 128256, 8192),
    "dozazen-tiny": uniform_config("dozazen-tiny", 3, 256, 4, 2, 64, 512, 128256, 96, (1, 2, 2)),
}


# ------------------------------------------------------------------- weights
@dataclasses.dataclass
class DozazenLayer:
    norms: List[Optional[torch.Tensor]]    # n1, n1b, n2, n2b: fp32 [Wp] (n2, n2b None without ffn)
    wqkv: torch.Tensor                     # [Hq DK + Hkv DK + Hkv DV, Wp], q / k rows half-rotated
    bqkv: torch.Tensor                     # fp32 [N]
    wo: torch.Tensor                       # [Wp, Hq DV]
    w_gate_up: Optional[torch.Tensor]      # [2 Fp, Wp], 16-row interleaved
    w_down: Optional[torch.Tensor]         # [Wp, Fp]


@dataclasses.dataclass
class DozazenWeights:
    embed: torch.Tensor                    # [V, Wp]
    layers: List[DozazenLayer]
    loop_in: Optional[torch.Tensor]        # [Wp, 2 Wp]
    final_norm: torch.Tensor               # fp32 [Wp]
    lm_head: torch.Tensor                  # [V padded to 4, Wp]


def half_rotation_order(dim: int, rot_dims: int, padded: int) -> torch.Tensor:
    """Row of the checkpoint's head that goes to each row of the padded head
    (-1: a zero row): pair (2i, 2i + 1) to (i, i + padded / 2), the dimensions
    that do not rotate to the rows left over."""
    at = torch.full((padded,), -1, dtype=torch.long)
    half = rot_dims // 2
    at[:half] = 2 * torch.arange(half)
    at[padded // 2:padded // 2 + half] = 2 * torch.arange(half) + 1
    free = (at < 0).nonzero().flatten()
    at[free[:dim - rot_dims]] = torch.arange(rot_dims, dim)
    return at


def pack_weights(cfg: DozazenConfig, get, device, dtype=torch.bfloat16) -> DozazenWeights:
    """Checkpoint tensors (``get(name)``) -> the kernels' layout on ``device``."""
    W = cfg.width
    Wp = _up(W, 64)

    def put(t):
        return t.to(dtype).contiguous().to(device)

    def vec(name):
        return _pad(get(name).float(), Wp).to(device)

    layers = []
    for i, s in enumerate(cfg.layer_specs):
        m, p = s.mixer, f"l{i}."
        DK, DV = head_size(m.dim), head_size(m.vdim)
        qk = half_rotation_order(m.dim, m.rot.dims, DK)
        vo = _leading(m.vdim, DV)
        parts = ((m.heads, m.dim, qk, "q"), (m.kv_heads, m.dim, qk, "k"), (m.kv_heads, m.vdim, vo, "v"))
        wqkv = torch.cat([_pick_rows(get(f"{p}mix.{n}"), h, d, o) for h, d, o, n in parts])
        bqkv = torch.cat([_pick_rows(get(f"{p}mix.{n}.b").float(), h, d, o) for h, d, o, n in parts])
        wo = _pick_rows(get(p + "mix.o").t(), m.heads, m.vdim, vo).t()
        gu = down = None
        if s.ffn is not None:
            Fp = _up(s.ffn, 64)
            gu = put(ref.interleave_gate_up(_pad(get(p + "mlp.gate"), Fp, Wp), _pad(get(p + "mlp.up"), Fp, Wp)))
            down = put(_pad(get(p + "mlp.down"), Wp, Fp))
        norms = [vec(p + "norm1"), vec(p + "norm1b")] + (
            [vec(p + "norm2"), vec(p + "norm2b")] if s.ffn is not None else [None, None])
        layers.append(DozazenLayer(norms, put(_pad(wqkv, wqkv.shape[0], Wp)), bqkv.contiguous().to(device),
                                   put(_pad(wo, Wp, wo.shape[1])), gu, down))
    loop_in = None
    if cfg.loop is not None:
        w = get("loop.in")
        loop_in = put(torch.cat([_pad(w[:, :W], Wp, Wp), _pad(w[:, W:], Wp, Wp)], dim=1))
    V = cfg.vocab_size
    return DozazenWeights(put(_pad(get("embed"), V, Wp)), layers, loop_in, vec("final.norm"),
                          put(_pad(get("head"), _up(V, 4), Wp)))


def tensor_shapes(cfg: DozazenConfig) -> Dict[str, Tuple[int, ...]]:
    """Checkpoint tensor names and shapes of ``cfg``."""
    W, V = cfg.width, cfg.vocab_size
    t: Dict[str, Tuple[int, ...]] = {"embed": (V, W), "final.norm": (W,), "head": (V, W)}
    if cfg.loop is not None:
        t["loop.in"] = (W, 2 * W)
    for i, s in enumerate(cfg.layer_specs):
        m, p = s.mixer, f"l{i}."
        t[p + "norm1"] = t[p + "norm1b"] = (W,)
        for n, rows in (("q", m.heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.kv_heads * m.vdim)):
            t[p + "mix." + n], t[p + f"mix.{n}.b"] = (rows, W), (rows,)
        t[p + "mix.o"] = (W, m.heads * m.vdim)
        if s.ffn is not None:
            t[p + "norm2"] = t[p + "norm2b"] = (W,)
            t[p + "mlp.gate"] = t[p + "mlp.up"] = (s.ffn, W)
            t[p + "mlp.down"] = (W, s.ffn)
    return t


def random_tensors(cfg: DozazenConfig, seed: int = 0, device="cpu"):
    """``get`` of random-init checkpoint tensors, each drawn when it is asked for."""
    shapes = tensor_shapes(cfg)
    index = {n: i for i, n in enumerate(shapes)}

    def get(name):
        shape = shapes[name]
        g = torch.Generator(device=device).manual_seed(seed * 1_000_003 + index[name])
        w = torch.randn(shape, generator=g, device=device)
        if len(shape) == 1:
            return w * 0.1 + (0.0 if name.endswith(".b") else 1.0)
        if name in ("embed",):
            return w / cfg.embed_scale
        return w * shape[1] ** -0.5
    return get


# --------------------------------------------------------------------- model
class DozazenModel:
    """Stateless forward over weights + an external paged KV cache."""

    tp = 1
    tp_rank = 0
    supports_cascade = False      # a shared prefix ends at a chunk's edge for every later query

    def __init__(self, cfg: DozazenConfig, weights: DozazenWeights, device):
        self.cfg, self.w, self.device = cfg, weights, torch.device(device)
        self.dtype = weights.embed.dtype
        self.runs = cfg.runs()
        mixers = [s.mixer for s in cfg.layer_specs]
        # (work-list sizing of the scheduler: the fewest key heads, the most query heads)
        self.hkv, self.hq = min(m.kv_heads for m in mixers), max(m.heads for m in mixers)
        self.kv_specs = [(m.kv_heads, head_size(m.dim), head_size(m.vdim))
                         for m in (mixers[i] for i, _ in self.runs)]
        tables: Dict[tuple, torch.Tensor] = {}
        self.cos_sin = []
        for m in mixers:
            key = (m.rot, head_size(m.dim))
            if key not in tables:
                tables[key] = self._table(*key)
            self.cos_sin.append(tables[key])
        self.logit_scale, self.logit_cap = cfg.logit_scale, cfg.logit_cap

    def _table(self, rot: Rotary, padded: int) -> torch.Tensor:
        return rope_table(rot, self.cfg.max_pos, padded // 2, self.device)

    @classmethod
    def random(cls, name, device, seed: int = 0, dtype=torch.bfloat16):
        cfg = name if isinstance(name, DozazenConfig) else CONFIGS[name]
        return cls(cfg, pack_weights(cfg, random_tensors(cfg, seed, device), device, dtype), device)

    def attended_keys(self, start: int, take: int) -> int:
        """Most keys one of the tokens at [start, start + take) sees in any layer."""
        best = 0
        for s in self.cfg.layer_specs:
            c = s.mixer.chunk
            best = max(best, start + take - (start // c * c if c else 0))
        return best

    # ------------------------------------------------------------- forward
    def forward(self, step, kv, tap=None) -> torch.Tensor:
        """One ragged step; final-normed hidden states of ``step.logit_rows``.
        ``tap(run, x)`` sees the residual stream after every layer run."""
        cfg, w, eps, W = self.cfg, self.w, self.cfg.eps, self.cfg.width
        T, Wp = step.token_ids.numel(), w.embed.shape[1]
        rows = step.logit_rows
        pair = left = None
        if cfg.loop is not None:                       # [x ; x0], the input of a pass
            pair = torch.empty(T, 2 * Wp, device=self.device, dtype=self.dtype)
            left = pair[:, :Wp]
        x = ops.embedding_scaled(step.token_ids, w.embed, cfg.embed_scale,
                                 None if pair is None else pair[:, Wp:])
        h = torch.empty(T, Wp, device=self.device, dtype=self.dtype)
        y = w_post = None                              # sublayer output the residual has not taken yet
        for r, (i, begins) in enumerate(self.runs):
            lw, m, last = w.layers[i], cfg.layer_specs[i].mixer, r + 1 == len(self.runs)
            n1, n1b, n2, n2b = lw.norms
            if begins:
                ops.residual_norm(x, W, eps, y, w_post, None, left)
                if tap is not None and r:
                    tap(r - 1, x[:, :W])
                x = ops.gemm_f32out(pair, w.loop_in)
                ops.residual_norm(x, W, eps, None, None, n1, h)
            else:
                ops.residual_norm(x, W, eps, y, w_post, n1, h)
                if tap is not None and r:
                    tap(r - 1, x[:, :W])
            kc, vc = kv.layer(r)
            q = torch.empty(T, m.heads, kc.shape[3], device=self.device, dtype=self.dtype)
            ops.qkv_rope_bias(h, lw.wqkv, lw.bqkv, step.positions, step.slots, self.cos_sin[i], q, kc, vc)
            if last and rows.numel() == 0 and tap is None:
                return h.new_empty(0, Wp)              # every key is in the cache; nothing is read
            a = ops.masked_attention(q, kc, vc, step.attn, m.scale, cfg.group, m.soft_cap,
                                     m.chunk, True)
            a = a.view(T, -1)
            if last and tap is None:                   # only the asked-for rows go on
                ri = rows.long()
                x, a = x.index_select(0, ri), a.index_select(0, ri)
                h = torch.empty(ri.numel(), Wp, device=self.device, dtype=self.dtype)
            y, w_post = ops.gemm(a, lw.wo), n1b
            if n2 is not None:
                ops.residual_norm(x, W, eps, y, w_post, n2, h)
                y, w_post = ops.gemm(ops.gemm_silu(h, lw.w_gate_up, act="gelu_tanh"), lw.w_down), n2b
        ops.residual_norm(x, W, eps, y, w_post, w.final_norm, h)
        if tap is not None:
            tap(len(self.runs) - 1, x[:, :W])
            h = h.index_select(0, rows.long())
        return h

    def logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """[R, vocab] fp32 logits of ``forward``'s rows."""
        z = ops.logit_finish(ops.gemm_f32out(hidden, self.w.lm_head), self.logit_scale, self.logit_cap)
        return z[:, :self.cfg.vocab_size]


# ------------------------------------------------------------------- loading
def load(path, device, dtype=torch.bfloat16, max_pos: Optional[int] = None) -> DozazenModel:
    """Model over a checkpoint directory (config.json + safetensors)."""
    from .weights import _Reader
    path = Path(path)
    cfg = config_from_json(json.loads((path / "config.json").read_text()), path.name,
                           MAX_POS if max_pos is None else max_pos)
    return DozazenModel(cfg, pack_weights(cfg, _Reader(path).full, device, dtype), device)


def save(cfg: DozazenConfig, get, path) -> None:
    """Checkpoint directory from tensors in the checkpoint layout (``get(name)``)."""
    from .weights import save_tensors
    save_tensors(path, tensor_shapes(cfg), get, config_to_json(cfg))
