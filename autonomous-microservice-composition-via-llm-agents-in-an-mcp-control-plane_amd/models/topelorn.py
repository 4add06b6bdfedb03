"""Topelorn decoder: attention and feed-forward side by side on one layer norm;
two kinds of attention, both windowed and gated per head; an fp32 residual stream.

One ragged, paged step (ln = layer norm without bias, rms = rms norm, both with
weights; f = the gated feed-forward, silu):

    x = embed(ids)                                          fp32 residual
    per layer:  h = ln(x);  x = x + mix(h) + f(h)
    logits = ln(x) embed^T

``mix`` of an attention layer, query head n of H, key position j of query i:

    q, k = rms per head of Wq h, Wk h;   v = (1 - lam) Wv h + lam v_first
    s = q . k scale - 2^(-8 (n + 1) / H) (i - j)            j <= i, i - j < window or j < keep_first
    a = sum_j e^s v / (e^sink_n + sum_j e^s);   Wo [a sigmoid(g_n . h)]

(v_first: the values of the first layer that mixes), of a latent layer:

    c = rms(Wc h), r = rot(Wr h): the cached row;  q = [qn | rot(qr)] of Wq h
    s = (qn . Wuk c + qr . r) scale,  values Wuv c, ordinary softmax, i - j < window

How it maps onto the shared machinery:

* all projections of h that feed the mixer, the head gates included, are ONE
  product (``w_in``); one kernel norms heads, mixes values and writes the cache;
* latent layers cache [c | r] and nothing else.  Decoding and short portions run
  absorbed: (Wuk^T qn) . c and Wuv (sum p c), one product per head on either side
  (``ops.gemm_heads``), attention on the cached rows as they are, keys and values
  at once, one key head for all query heads.  Long portions expand the latents of
  the keys they see (one product) and run plain attention per head
  (``ops.latent_prefill``): less arithmetic once enough queries share a key;
* the feed-forward's down product takes the mixer's output as its residual, so a
  layer adds one vector to the stream, in the pass that also norms it for the
  next layer (``ops.residual_norm``);
* every size is padded with zero rows / columns, which is exact.

``dtype`` float32 weights run everything in 32 bits, the caches included.
"""
from __future__ import annotations

import dataclasses
import json
from pathlib import Path
from typing import Dict, List, Optional, Tuple, Union

import torch

from .. import ops
from ..engine.batch import long_spans
from ..ops import reference as ref
from .llama import padded_group
from .packing import MAX_POS, Rotary, head_size, leading, pad, pick_rows, rope_table, up


@dataclasses.dataclass(frozen=True)
class WindowAttention:
    heads: int
    kv_heads: int
    dim: int                  # query / key head size
    vdim: int                 # value head size
    window: int               # keys a query sees, its own included (0: all)
    keep_first: int           # first keys of the sequence that every query sees
    scale: float
    v_mix: bool

    # padded sizes
    @property
    def dk(self) -> int:
        return head_size(self.dim)

    @property
    def dv(self) -> int:
        return head_size(self.vdim)

    @property
    def kv_spec(self):
        return self.kv_heads, self.dk, self.dv


@dataclasses.dataclass(frozen=True)
class LatentAttention:
    heads: int
    dim: int                  # unrotated query / key size per head
    rot_dim: int              # rotated size, the key part shared by the heads
    vdim: int
    kv_rank: int
    window: int
    scale: float
    rot: Rotary

    keep_first = 0

    # padded sizes: the query's parts, the latent, (cached row, values' columns of it)
    @property
    def dim_p(self) -> int:
        return up(self.dim, 32)

    @property
    def rot_p(self) -> int:
        return up(self.rot_dim, 16)

    @property
    def rank_p(self) -> int:
        return up(self.kv_rank, 16)

    @property
    def row(self) -> Tuple[int, int]:
        need = self.rank_p + self.rot_p
        return next(((k, v) for k, v in ops.LATENT_SIZES if k >= need and v >= self.kv_rank),
                    (up(need, 64), up(self.kv_rank, 64)))

    @property
    def vdim_p(self) -> int:
        return head_size(self.vdim)

    @property
    def expands(self) -> bool:
        """Keys and values of a head fit the expanded form."""
        return max(self.dim_p + self.rot_p, self.vdim_p) <= ops.MASKED_MAX_HEAD

    @property
    def kv_spec(self):
        return 1, self.row[0], 0


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: Union[WindowAttention, LatentAttention]
    ffn: Optional[int]        # feed-forward width, None: no feed-forward

    @property
    def latent(self) -> bool:
        return isinstance(self.mixer, LatentAttention)


@dataclasses.dataclass(frozen=True)
class TopelornConfig:
    name: str
    vocab_size: int
    width: int
    layer_specs: Tuple[LayerSpec, ...]
    eps: float = 1e-5
    max_pos: int = MAX_POS

    @property
    def layers(self) -> int:
        return len(self.layer_specs)

    @property
    def hidden(self) -> int:
        return self.width

    @property
    def group(self) -> int:
        """Query heads per key head the attention work items are cut for: the
        smallest of the layers (larger groups walk several row tiles)."""
        return min(padded_group(min(s.mixer.heads // s.mixer.kv_spec[0], 16)) for s in self.layer_specs)

    def first_mixed(self) -> Optional[int]:
        """The layer whose values later layers mix in."""
        return next((i for i, s in enumerate(self.layer_specs) if not s.latent and s.mixer.v_mix), None)

    def params(self) -> int:
        n = 0
        for shape in tensor_shapes(self).values():
            k = 1
            for d in shape:
                k *= d
            n += k
        return n


def config_from_json(c: dict, name: str = "topelorn", max_pos: int = MAX_POS) -> TopelornConfig:
    specs = []
    for i, ly in enumerate(c["layers"]):
        m, mlp = ly["mixer"], ly.get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise NotImplementedError(f"layer {i}: feed-forward kind {mlp['kind']!r}")
        mask = m.get("mask") or {}
        window = int(mask.get("size") or 0)
        if ly["type"] == "attention":
            if m["heads"] % m["kv_heads"]:
                raise ValueError(f"layer {i}: {m['heads']} query heads on {m['kv_heads']} key heads")
            mixer = WindowAttention(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]),
                                    window, int(mask.get("keep_first") or 0), float(m["scale"]),
                                    bool(m.get("v_mix")))
        elif ly["type"] == "latent_attention":
            r = m["rot"]
            if r["dims"] % 2 or r["dims"] > m["rot_dim"]:
                raise ValueError(f"layer {i}: rotated dimensions {r['dims']} of {m['rot_dim']}")
            if mask.get("keep_first"):
                raise NotImplementedError(f"layer {i}: kept first tokens of a latent layer")
            mixer = LatentAttention(int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]),
                                    int(m["kv_rank"]), window, float(m["scale"]),
                                    Rotary(int(r["dims"]), float(r["base"])))
        else:
            raise NotImplementedError(f"layer {i}: mixer type {ly['type']!r}")
        specs.append(LayerSpec(mixer, None if mlp is None else int(mlp["ff"])))
    mixed = {(s.mixer.kv_heads, s.mixer.vdim) for s in specs if not s.latent and s.mixer.v_mix}
    if len(mixed) > 1:
        raise ValueError(f"layers that mix values have unequal value heads: {sorted(mixed)}")
    return TopelornConfig(name, int(c["vocab"]), int(c["width"]), tuple(specs), float(c["norm"]["eps"]), max_pos)


def config_to_json(cfg: TopelornConfig) -> dict:
    layers = []
    for s in cfg.layer_specs:
        m = s.mixer
        if s.latent:
            d = {"heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim, "kv_rank": m.kv_rank,
                 "mask": {"size": m.window}, "rot": {"dims": m.rot.dims, "base": m.rot.base}}
        else:
            d = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "v_mix": m.v_mix,
                 "mask": {"size": m.window, "keep_first": m.keep_first}}
        layers.append({"type": "latent_attention" if s.latent else "attention", "mixer": {**d, "scale": m.scale},
                       "mlp": None if s.ffn is None else {"kind": "dense", "ff": s.ffn}})
    return {"architecture": "Topelorn", "vocab": cfg.vocab_size, "width": cfg.width, "layers": layers,
            "norm": {"eps": cfg.eps}}


def alternating_config(name: str, layers: int, width: int, heads: int, kv_heads: int, dim: int, ffn: int,
                       vocab_size: int, window: int = 4096, keep_first: int = 4, kv_rank: int = 512,
                       rot_dim: int = 64, latent_every: int = 2, **kw) -> TopelornConfig:
    """Equal sizes, every ``latent_every``-th layer latent (benchmarks, tests,
    named random-init models)."""
    attn = WindowAttention(heads, kv_heads, dim, dim, window, keep_first, dim ** -0.5, True)
    lat = LatentAttention(heads, dim, rot_dim, dim, kv_rank, window, (dim + rot_dim) ** -0.5,
                          Rotary(rot_dim, 500000.0))
    specs = tuple(LayerSpec(lat if (i + 1) % latent_every == 0 else attn, ffn) for i in range(layers))
    return TopelornConfig(name, vocab_size, width, specs, **kw)


CONFIGS: Dict[str, TopelornConfig] = {
    # the layer sizes of an 8B model
    "topelorn-8b": alternating_config("topelorn-8b", 32, 4096, 32, 8, 128, 14336, 128256),
    "topelorn-8b-2l": alternating_config("topelorn-8b-2l", 2, 4096, 32, 8, 128, 14336, 128256),
    "topelorn-tiny": alternating_config("topelorn-tiny", 4, 256, 4, 2, 64, 512, 128256, window=96,
                                        keep_first=3, kv_rank=64, rot_dim=32),
}


# ------------------------------------------------------------------- weights
@dataclasses.dataclass
class TopelornLayer:
    norm: torch.Tensor                     # fp32 [Wp]
    w_in: torch.Tensor                     # [N, Wp]: q | k | v | gates, or q | latent, rotated key | gates
    wo: torch.Tensor                       # [Wp, H * value size]
    w_gate_up: Optional[torch.Tensor]      # [2 Fp, Wp], 16-row interleaved
    w_down: Optional[torch.Tensor]         # [Wp, Fp]
    # attention layers
    q_norm: Optional[torch.Tensor] = None  # fp32 [DK]
    k_norm: Optional[torch.Tensor] = None
    sinks: Optional[torch.Tensor] = None   # fp32 [H]
    lam: float = 0.0                       # weight of the first mixed layer's values
    # latent layers
    c_norm: Optional[torch.Tensor] = None  # fp32 [latent]
    w_uk: Optional[torch.Tensor] = None    # [H, latent, dim]: the absorbed query's product
    w_uv: Optional[torch.Tensor] = None    # [H, value size, DV]
    w_ukv: Optional[torch.Tensor] = None   # [H (dim + value size), latent to 64]: expands latents


@dataclasses.dataclass
class TopelornWeights:
    embed: torch.Tensor                    # [V padded to 4, Wp]
    layers: List[TopelornLayer]
    final_norm: torch.Tensor               # fp32 [Wp]

    @property
    def lm_head(self) -> torch.Tensor:     # tied
        return self.embed


def pack_weights(cfg: TopelornConfig, get, device, dtype=torch.bfloat16) -> TopelornWeights:
    """Checkpoint tensors (``get(name)``) -> the kernels' layout on ``device``."""
    W = cfg.width
    Wp = up(W, 64)
    first = cfg.first_mixed()

    def put(t):
        return t.to(dtype).contiguous().to(device)

    def vec(name, n):
        return pad(get(name).float(), n).to(device)

    def columns(w, heads, dim, order):
        return pick_rows(w.t(), heads, dim, order).t()

    layers = []
    for i, s in enumerate(cfg.layer_specs):
        m, p = s.mixer, f"l{i}."
        gates = pad(get(p + "mix.g"), up(m.heads, 16), W)
        kw = {}
        if s.latent:
            vo = leading(m.vdim, m.vdim_p)
            qo = torch.cat([leading(m.dim, m.dim_p),
                            torch.where((t := leading(m.rot_dim, m.rot_p)) >= 0, t + m.dim, t)])
            down = get(p + "mix.dkv")
            rows = [pick_rows(get(p + "mix.q"), m.heads, m.dim + m.rot_dim, qo),
                    pad(down[:m.kv_rank], m.rank_p, W), pad(down[m.kv_rank:], m.rot_p, W), gates]
            uk = get(p + "mix.uk").view(m.heads, m.dim, m.kv_rank).transpose(1, 2)
            uv = get(p + "mix.uv").view(m.heads, m.vdim, m.kv_rank)
            kw = dict(c_norm=vec(p + "mix.dkv.norm", m.rank_p),
                      w_uk=put(pad(uk, m.heads, m.rank_p, m.dim_p)),
                      w_uv=put(pad(uv, m.heads, m.vdim_p, m.row[1])))
            if m.expands and dtype == torch.bfloat16:
                k64 = up(m.rank_p, 64)
                ukv = torch.cat([pad(uk.transpose(1, 2), m.heads, m.dim_p, k64), pad(uv, m.heads, m.vdim_p, k64)], 1)
                kw["w_ukv"] = put(ukv.reshape(-1, k64))
        else:
            qk, vo = leading(m.dim, m.dk), leading(m.vdim, m.dv)
            rows = [pick_rows(get(p + "mix.q"), m.heads, m.dim, qk),
                    pick_rows(get(p + "mix.k"), m.kv_heads, m.dim, qk),
                    pick_rows(get(p + "mix.v"), m.kv_heads, m.vdim, vo), gates]
            kw = dict(q_norm=vec(p + "mix.q.norm", m.dk), k_norm=vec(p + "mix.k.norm", m.dk),
                      sinks=vec(p + "mix.sink", m.heads),
                      lam=float(get(p + "mix.vmix")) if m.v_mix and i != first else 0.0)
        w_in = torch.cat(rows)
        wo = columns(get(p + "mix.o"), m.heads, m.vdim, vo)
        gu = down = None
        if s.ffn is not None:
            Fp = up(s.ffn, 64)
            gu = put(ref.interleave_gate_up(pad(get(p + "mlp.gate"), Fp, Wp), pad(get(p + "mlp.up"), Fp, Wp)))
            down = put(pad(get(p + "mlp.down"), Wp, Fp))
        layers.append(TopelornLayer(vec(p + "norm1", Wp), put(pad(w_in, w_in.shape[0], Wp)),
                                    put(pad(wo, Wp, wo.shape[1])), gu, down, **kw))
    return TopelornWeights(put(pad(get("embed"), up(cfg.vocab_size, 4), Wp)), layers, vec("final.norm", Wp))


def tensor_shapes(cfg: TopelornConfig) -> Dict[str, Tuple[int, ...]]:
    """Checkpoint tensor names and shapes of ``cfg``."""
    W = cfg.width
    t: Dict[str, Tuple[int, ...]] = {"embed": (cfg.vocab_size, W), "final.norm": (W,)}
    for i, s in enumerate(cfg.layer_specs):
        m, p = s.mixer, f"l{i}."
        t[p + "norm1"] = (W,)
        if s.latent:
            t[p + "mix.q"] = (m.heads * (m.dim + m.rot_dim), W)
            t[p + "mix.dkv"] = (m.kv_rank + m.rot_dim, W)
            t[p + "mix.dkv.norm"] = (m.kv_rank,)
            t[p + "mix.uk"] = (m.heads * m.dim, m.kv_rank)
            t[p + "mix.uv"] = (m.heads * m.vdim, m.kv_rank)
        else:
            for n, rows in (("q", m.heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.kv_heads * m.vdim)):
                t[p + "mix." + n] = (rows, W)
            t[p + "mix.q.norm"] = t[p + "mix.k.norm"] = (m.dim,)
            if m.v_mix:
                t[p + "mix.vmix"] = ()
            t[p + "mix.sink"] = (m.heads,)
        t[p + "mix.g"] = (m.heads, W)
        t[p + "mix.o"] = (W, m.heads * m.vdim)
        if s.ffn is not None:
            t[p + "mlp.gate"] = t[p + "mlp.up"] = (s.ffn, W)
            t[p + "mlp.down"] = (W, s.ffn)
    return t


def random_tensors(cfg: TopelornConfig, seed: int = 0, device="cpu"):
    """``get`` of random-init checkpoint tensors, each drawn when it is asked for."""
    shapes = tensor_shapes(cfg)
    index = {n: i for i, n in enumerate(shapes)}

    def get(name):
        shape = shapes[name]
        g = torch.Generator(device=device).manual_seed(seed * 1_000_003 + index[name])
        w = torch.randn(shape, generator=g, device=device)
        if name.endswith(".sink"):
            return w
        if len(shape) < 2:                             # norms around 1, mixing weights around 1/2
            return w * 0.1 + (1.0 if shape else 0.5)
        return w if name == "embed" else w * shape[1] ** -0.5
    return get


# --------------------------------------------------------------------- model
class TopelornModel:
    """Stateless forward over weights + an external paged KV cache."""

    tp = 1
    tp_rank = 0
    supports_cascade = False      # a shared prefix leaves the window as a request goes on
    uses_host_step = True         # spans this long expand the latents they see
    EXPAND_MIN, EXPAND_MAX_BYTES = 192, 4 << 30
    logit_scale, logit_cap = 1.0, 0.0

    def __init__(self, cfg: TopelornConfig, weights: TopelornWeights, device):
        self.cfg, self.w, self.device = cfg, weights, torch.device(device)
        self.dtype = weights.embed.dtype
        mixers = [s.mixer for s in cfg.layer_specs]
        self.kv_specs = [m.kv_spec for m in mixers]
        # (work-list sizing of the scheduler: the fewest key heads, the most query heads)
        self.hkv, self.hq = min(h for h, _, _ in self.kv_specs), max(m.heads for m in mixers)
        self.first = cfg.first_mixed()
        slopes, tables = {}, {}
        self.slopes, self.cos_sin = [], []
        for s in cfg.layer_specs:
            m = s.mixer
            if s.latent:
                if m.rot not in tables:
                    tables[m.rot] = rope_table(m.rot, cfg.max_pos, m.rot.dims // 2, self.device)
            elif m.heads not in slopes:
                n = torch.arange(1, m.heads + 1, dtype=torch.float64)
                slopes[m.heads] = torch.exp2(-8.0 * n / m.heads).float().to(self.device)
            self.cos_sin.append(tables[m.rot] if s.latent else None)
            self.slopes.append(None if s.latent else slopes[m.heads])

    @classmethod
    def random(cls, name, device, seed: int = 0, dtype=torch.bfloat16):
        cfg = name if isinstance(name, TopelornConfig) else CONFIGS[name]
        return cls(cfg, pack_weights(cfg, random_tensors(cfg, seed, device), device, dtype), device)

    def attended_keys(self, start: int, take: int) -> int:
        """Most keys one of the tokens at [start, start + take) sees in any layer,
        with the tokens of the span around it."""
        return max(min(start + take, m.window + take + m.keep_first) if m.window else start + take
                   for m in (s.mixer for s in self.cfg.layer_specs))

    # ------------------------------------------------------------- forward
    def forward(self, step, kv, tap=None) -> torch.Tensor:
        """One ragged step; final-normed hidden states of ``step.logit_rows``.
        ``tap(layer, x)`` sees the residual stream after every layer."""
        cfg, w, eps, W = self.cfg, self.w, self.cfg.eps, self.cfg.width
        rows = step.logit_rows
        x = ops.embedding_scaled(step.token_ids, w.embed, 1.0)
        h = torch.empty(x.shape, device=self.device, dtype=self.dtype)
        y = v_first = None                             # the last layer's output; the mixed-in values
        for i, s in enumerate(cfg.layer_specs):
            lw, last = w.layers[i], i + 1 == cfg.layers
            ops.residual_norm(x, W, eps, y, None, lw.norm, h, center=True)
            if tap is not None and i:
                tap(i - 1, x[:, :W])
            z = ops.gemm(h, lw.w_in)
            a, v = (self._latent if s.latent else self._attention)(
                i, z, step, kv, v_first, last and rows.numel() == 0 and tap is None)
            if a is None:
                return h.new_empty(0, h.shape[1])      # every key is in the cache; nothing is read
            if i == self.first:
                v_first = v
            early = last and tap is None and rows.numel() < h.shape[0] and h.shape[0] > 64
            if early:                                  # only the asked-for rows go on (few tokens: all do)
                ri = rows.long()
                x, h, a = x.index_select(0, ri), h.index_select(0, ri), a.index_select(0, ri)
            y = ops.gemm(a, lw.wo)
            if s.ffn is not None:
                y = ops.gemm(ops.gemm_silu(h, lw.w_gate_up), lw.w_down, R=y)
        h = ops.residual_norm(x, W, eps, y, None, w.final_norm, torch.empty_like(h), center=True)
        if tap is not None:
            tap(cfg.layers - 1, x[:, :W])
        return h if early else h.index_select(0, rows.long())

    def _gates(self, m, z):
        return z[:, z.shape[1] - up(m.heads, 16):][:, :m.heads]

    def _attention(self, i, z, step, kv, v_first, cache_only):
        """([T, heads * value size] gated outputs, the projected values) of an
        attention layer on its projected rows ``z``."""
        m, lw, T = self.cfg.layer_specs[i].mixer, self.w.layers[i], z.shape[0]
        kc, vc = kv.layer(i)
        q = torch.empty(T, m.heads, m.dk, device=self.device, dtype=self.dtype)
        ops.qk_norm_kv(z, step.slots, lw.q_norm, lw.k_norm, m.dim, self.cfg.eps, q, kc, vc,
                       v_first if m.v_mix else None, lw.lam)
        if cache_only:
            return None, None
        a = ops.masked_attention(q, kc, vc, step.attn, m.scale, self.cfg.group, sink=lw.sinks, window=m.window,
                                 keep_first=m.keep_first, slopes=self.slopes[i], gate=self._gates(m, z))
        at = (m.heads + m.kv_heads) * m.dk
        return a.view(T, -1), z[:, at:at + m.kv_heads * m.dv]

    def _latent(self, i, z, step, kv, v_first, cache_only):
        """(gated outputs, None) of a latent layer."""
        m, lw, T = self.cfg.layer_specs[i].mixer, self.w.layers[i], z.shape[0]
        kc, _ = kv.layer(i)
        plan = self._plan(i, step)
        lo, hi = (0, T) if plan is None else plan.rest or (0, 0)      # tokens that run absorbed
        q = torch.empty(T, m.heads, m.row[0], device=self.device, dtype=self.dtype) \
            if hi > lo and not cache_only else None
        ops.latent_qkv(z, step.positions, step.slots, self.cos_sin[i], lw.c_norm, self.cfg.eps, m.heads,
                       m.dim_p, m.rot_p, m.rank_p, m.kv_rank, q, kc)
        if cache_only:
            return None, None
        out = torch.empty(T, m.heads, m.vdim_p, device=self.device, dtype=self.dtype)
        if q is not None:
            per = m.dim_p + m.rot_p
            qn = z[:, :m.heads * per].view(T, m.heads, per)[..., :m.dim_p]
            ops.gemm_heads(qn[lo:hi], lw.w_uk, q[lo:hi, :, :m.rank_p])
            a = ops.masked_attention(q, kc, None, step.attn, m.scale, self.cfg.group, window=m.window,
                                     gate=self._gates(m, z), v_dim=m.row[1],
                                     skip_q=0 if plan is None else self.EXPAND_MIN)
            ops.gemm_heads(a[lo:hi], lw.w_uv, out[lo:hi])
        if plan is not None:
            c = torch.empty(plan.pages.numel() * kc.shape[2], lw.w_ukv.shape[1], device=self.device, dtype=self.dtype)
            ops.latent_gather(kc, plan.pages, plan.valid, m.rank_p, c)
            ops.latent_prefill(z, step.attn, plan, step.positions, self.cos_sin[i], m.heads, m.dim_p, m.rot_p,
                               ops.gemm(c, lw.w_ukv), kc, m.rank_p, m.scale, m.window, self._gates(m, z), out)
        return out.view(T, -1), None

    def _plan(self, i, step):
        """The spans of the step whose keys layer ``i`` expands (one plan per
        window, kept with the step)."""
        m, meta = self.cfg.layer_specs[i].mixer, step.attn
        if meta.host is None or self.w.layers[i].w_ukv is None or self.device.type != "cuda":
            return None
        plans = meta.host.plans
        if m.window not in plans:
            plans[m.window] = long_spans(meta.host, self.EXPAND_MIN, m.window, ops.LATENT_ITEM, self.device)
        plan = plans[m.window]
        if plan is None or plan.pages.numel() * 64 * self.w.layers[i].w_ukv.shape[0] * 2 > self.EXPAND_MAX_BYTES:
            return None
        return plan

    def logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """[R, vocab] fp32 logits of ``forward``'s rows."""
        return ops.gemm_f32out(hidden, self.w.lm_head)[:, :self.cfg.vocab_size]


# ------------------------------------------------------------------- loading
def load(path, device, dtype=torch.bfloat16, max_pos: Optional[int] = None) -> TopelornModel:
    """Model over a checkpoint directory (config.json + safetensors)."""
    from .weights import _Reader
    path = Path(path)
    cfg = config_from_json(json.loads((path / "config.json").read_text()), path.name,
                           MAX_POS if max_pos is None else max_pos)
    return TopelornModel(cfg, pack_weights(cfg, _Reader(path).full, device, dtype), device)


def save(cfg: TopelornConfig, get, path) -> None:
    """Checkpoint directory from tensors in the checkpoint layout (``get(name)``)."""
    from .weights import save_tensors
    save_tensors(path, tensor_shapes(cfg), get, config_to_json(cfg))
