"""Llama-3 decoder (the on-node planner LLM).

Replaces the reference's remote ``openai.ChatCompletion`` call
(control_plane.py:69-73).  Shapes are Meta's public Llama-3 configs (8B / 70B);
weights are random-init (no checkpoints are reachable here
north star) or loaded from safetensors (``models.weights``).

Forward of one ragged, paged step - every op is a gfx950 HIP
kernel from ``ops`` on GPU:

    x = embed(ids)                                   K8
    per layer:  h = rmsnorm(x)                       K3
                qkv = h Wqkv^T                       K1 (MFMA GEMM)
                q, K/V cache <- rope(qkv)            K4 + K10
                a = paged_attention(q, K, V)         K5/K6
                x = x + a Wo^T      (residual fused in the GEMM epilogue)
                [all-reduce over TP ranks]           C1 (RCCL / xGMI)
                h = rmsnorm(x); g = silu(h Wg^T) * (h Wu^T)   K1 with K7 fused
                x = x + g Wd^T      (fused residual) [all-reduce]  C2
    h_last = rmsnorm(x[rows that need a token])

Tensor parallelism is Megatron 1-D: Wqkv / Wgate|up column-parallel (whole
heads / FFN slices per rank), Wo / Wdown row-parallel followed by an
all-reduce; embeddings and the LM head are replicated (the constrained sampler
only touches a few LM-head rows, so every rank samples identically and no
logit collective is needed).

Sequence parallelism (Megatron SP; ``seq_parallel=True`` or
``MCP_SEQ_PARALLEL=1``, TP > 1 only): the residual stream is split by rows
across the TP ranks.  Each all-reduce after Wo / Wdown becomes a
reduce-scatter, and the residual add + RMSNorm run fused (``add_rmsnorm``, K3)
on this rank's T/tp rows.  Then an all-gather rebuilds the normed [T, H]
input of the next column-parallel GEMM.  The bytes moved are those of the
all-reduce.  The per-rank residual and norm traffic drops by tp.  The last
layer gathers the residual once and takes the row-selected path above.
"""
from __future__ import annotations

import dataclasses
import math
import os
from typing import List, Optional

import torch

from .. import ops
from ..ops import reference as ref

# Infinity Cache weight prefetch beside the decode attention (measured A/B:
# profiles/config2_decode_gemm_r4_ab.txt): on/off, largest step (tokens),
# bytes read per layer (o-projection first, then the head of gate|up), grid
_PF_ON = os.environ.get("MCP_WEIGHT_PREFETCH", "0") == "1"
_PF_MAX_T = int(os.environ.get("MCP_WEIGHT_PREFETCH_MAX_T", "64"))
# TP > 1, steps of at least this many tokens: the o-projection / MLP block
# runs as two row chunks whose all-reduces go out on a comm stream under the
# other chunk's GEMMs (_mlp_block_overlapped); 0 (default) disables.
# Measured on one GPU with every all-reduce emulated (bench_tp.py
# --simulate-rank 8 --emulate-comm, profiles/config4_tp8_overlap_emulated_r5.jsonl):
# 71.2 plans/s chunked vs 76.2 in line - the half-M GEMMs lose ~15 % and a
# K12-sized comm kernel holds up to half the CUs the other chunk's GEMMs need
_TP_OVERLAP_MIN_T = int(os.environ.get("MCP_TP_OVERLAP_MIN_T", "0"))
_PF_BYTES = int(float(os.environ.get("MCP_WEIGHT_PREFETCH_MB", "64")) * (1 << 20))
_PF_WGS = int(os.environ.get("MCP_WEIGHT_PREFETCH_WGS", "256"))


@dataclasses.dataclass(frozen=True)
class LlamaConfig:
    name: str
    vocab_size: int = 128256
    hidden: int = 4096
    layers: int = 32
    heads: int = 32
    kv_heads: int = 8
    head_dim: int = 128
    ffn: int = 14336
    rope_theta: float = 500000.0
    eps: float = 1e-5
    max_pos: int = 8192
    # Llama-3.1 rope scaling: (factor, low_freq_factor, high_freq_factor,
    # original_max_position_embeddings); None = plain RoPE (Llama-3)
    rope_scaling: Optional[tuple] = None
    # GQA padding: the checkpoint has q_heads_true query heads (group not a
    # divisor of 16, e.g. Llama-3.2-3B's 24 q / 8 kv = 3); the engine runs
    # ``heads`` = kv_heads x (group rounded up to a divisor of 16) with
    # all-zero Wq rows / Wo columns in the pad heads, which is exact: a pad
    # head's attention output only meets zero columns of Wo.  0 = no padding.
    q_heads_true: int = 0
    tie_embeddings: bool = False

    @property
    def group(self) -> int:
        return self.heads // self.kv_heads

    @property
    def group_true(self) -> int:
        return (self.q_heads_true or self.heads) // self.kv_heads

    def params(self) -> int:
        H, D, hq = self.hidden, self.head_dim, self.q_heads_true or self.heads
        per_layer = H * (hq + 2 * self.kv_heads) * D + hq * D * H + 3 * H * self.ffn + 2 * H
        return self.layers * per_layer + (1 if self.tie_embeddings else 2) * self.vocab_size * H + H

    def kv_bytes_per_token(self, tp: int = 1) -> int:
        """bf16 K + V bytes one token occupies in the paged cache of one TP rank."""
        return self.layers * 2 * (self.kv_heads // tp) * self.head_dim * 2


def padded_group(group: int) -> int:
    """Smallest divisor of 16 (the MFMA row count attention packs heads into)
    that is >= ``group``."""
    for g in (1, 2, 4, 8, 16):
        if g >= group:
            return g
    raise ValueError(f"GQA group {group} > 16")


def pad_gqa(cfg: "LlamaConfig") -> "LlamaConfig":
    """Config with query heads padded so the GQA group divides 16 (identity
    when it already does)."""
    g = cfg.heads // cfg.kv_heads
    gp = padded_group(g)
    if gp == g:
        return cfg
    return dataclasses.replace(cfg, heads=cfg.kv_heads * gp, q_heads_true=cfg.heads)


def pad_q_rows(w: torch.Tensor, cfg: "LlamaConfig") -> torch.Tensor:
    """[q_heads_true*D, H] -> [heads*D, H] with zero pad heads at the end of
    each kv group (full, unsharded tensors)."""
    if not cfg.q_heads_true:
        return w
    D, kv = cfg.head_dim, cfg.kv_heads
    x = w.reshape(kv, cfg.group_true, D, -1)
    out = x.new_zeros(kv, cfg.group, D, x.shape[-1])
    out[:, :cfg.group_true] = x
    return out.reshape(cfg.heads * D, -1)


def pad_o_cols(w: torch.Tensor, cfg: "LlamaConfig") -> torch.Tensor:
    """[H, q_heads_true*D] -> [H, heads*D] (zero columns for the pad heads)."""
    return w if not cfg.q_heads_true else pad_q_rows(w.t().contiguous(), cfg).t().contiguous()


def unpad_q_rows(w: torch.Tensor, cfg: "LlamaConfig") -> torch.Tensor:
    if not cfg.q_heads_true:
        return w
    D = cfg.head_dim
    return w.reshape(cfg.kv_heads, cfg.group, D, -1)[:, :cfg.group_true].reshape(
        cfg.q_heads_true * D, -1).contiguous()


def unpad_o_cols(w: torch.Tensor, cfg: "LlamaConfig") -> torch.Tensor:
    return w if not cfg.q_heads_true else unpad_q_rows(w.t().contiguous(), cfg).t().contiguous()


_LLAMA31_ROPE = (8.0, 1.0, 4.0, 8192)

CONFIGS = {
    "llama3-8b": LlamaConfig("llama3-8b"),
    "llama3-70b": LlamaConfig("llama3-70b", hidden=8192, layers=80, heads=64, kv_heads=8, ffn=28672),
    # Llama-3.1: same shapes, 128k context through rope scaling (only the
    # host-built cos/sin table changes; the kernels are shared)
    "llama3.1-8b": LlamaConfig("llama3.1-8b", max_pos=131072, rope_scaling=_LLAMA31_ROPE),
    "llama3.1-70b": LlamaConfig("llama3.1-70b", hidden=8192, layers=80, heads=64, kv_heads=8,
                                ffn=28672, max_pos=131072, rope_scaling=_LLAMA31_ROPE),
    # Llama-3.2-3B: 24 q / 8 kv heads (group 3) padded to 32 q heads, tied
    # embeddings, rope scaling factor 32
    "llama3.2-3b": LlamaConfig("llama3.2-3b", hidden=3072, layers=28, heads=32, kv_heads=8,
                               ffn=8192, max_pos=131072, rope_scaling=(32.0, 1.0, 4.0, 8192),
                               q_heads_true=24, tie_embeddings=True),
    # reduced configs with the same kernels (tests / smoke): head_dim stays 128
    "llama3-1b-ish": LlamaConfig("llama3-1b-ish", hidden=2048, layers=16, heads=16, kv_heads=4, ffn=8192),
    "tiny": LlamaConfig("tiny", hidden=256, layers=2, heads=2, kv_heads=1, ffn=512),
    # Llama-3-8B layer shapes, 2 layers: tests of shape-specific kernels
    # (the fused decode attention + o-projection needs K = Hq D = 4096)
    "llama3-8b-2l": LlamaConfig("llama3-8b-2l", layers=2),
    "tiny-tp": LlamaConfig("tiny-tp", hidden=512, layers=2, heads=4, kv_heads=2, ffn=1024),
    # 8 KV heads: shards to TP = 8 like the 70B (one KV head per rank)
    "tiny-tp8": LlamaConfig("tiny-tp8", hidden=2048, layers=2, heads=16, kv_heads=8, ffn=4096),
}


def get_config(name: str) -> LlamaConfig:
    if name not in CONFIGS:
        raise KeyError(f"unknown model config {name!r}; have {sorted(CONFIGS)}")
    return CONFIGS[name]


@dataclasses.dataclass
class LayerWeights:
    attn_norm: torch.Tensor
    wqkv: torch.Tensor        # [(Hq + 2 Hkv) * D / tp, H]
    wo: torch.Tensor          # [H, Hq * D / tp]
    mlp_norm: torch.Tensor
    w_gate_up: torch.Tensor   # [2 F / tp, H]  gate/up rows interleaved in 16-row groups
    w_down: torch.Tensor      # [H, F / tp]


@dataclasses.dataclass
class LlamaWeights:
    embed: torch.Tensor       # [V, H] (replicated)
    layers: List[LayerWeights]
    final_norm: torch.Tensor
    lm_head: torch.Tensor     # [V, H] (replicated)


def shard_rows(w: torch.Tensor, rank: int, tp: int) -> torch.Tensor:
    n = w.shape[0] // tp
    return w[rank * n:(rank + 1) * n].contiguous()


def shard_cols(w: torch.Tensor, rank: int, tp: int) -> torch.Tensor:
    n = w.shape[1] // tp
    return w[:, rank * n:(rank + 1) * n].contiguous()


def shard_layer(full: LayerWeights, cfg: LlamaConfig, rank: int, tp: int) -> LayerWeights:
    """Megatron split of one full layer (used by tests and the safetensors loader)."""
    D = cfg.head_dim
    q, k, v = torch.split(full.wqkv, [cfg.heads * D, cfg.kv_heads * D, cfg.kv_heads * D])
    wqkv = torch.cat([shard_rows(q, rank, tp), shard_rows(k, rank, tp), shard_rows(v, rank, tp)])
    g, u = ref.deinterleave_gate_up(full.w_gate_up)
    return LayerWeights(attn_norm=full.attn_norm, wqkv=wqkv.contiguous(),
                        wo=shard_cols(full.wo, rank, tp), mlp_norm=full.mlp_norm,
                        w_gate_up=ref.interleave_gate_up(shard_rows(g, rank, tp),
                                                         shard_rows(u, rank, tp)).contiguous(),
                        w_down=shard_cols(full.w_down, rank, tp))


def random_weights(cfg: LlamaConfig, device, dtype=torch.bfloat16, seed: int = 0, tp_rank: int = 0,
                   tp: int = 1, std: float = 0.02) -> LlamaWeights:
    """Random-init weights, generated shard-locally on the target device.

    Each rank draws its own shard (70B at TP=8 never materialises the full
    tensors).  Replicated tensors use a rank-independent seed."""
    dev = torch.device(device)
    g = torch.Generator(device=dev)
    D, H = cfg.head_dim, cfg.hidden

    def rnd(shape, s, scale=std):
        g.manual_seed(s)
        return (torch.randn(shape, generator=g, device=dev, dtype=torch.float32) * scale).to(dtype)

    def norm_w():
        return torch.ones(H, device=dev, dtype=dtype)

    base = seed * 1_000_003
    layers = []
    hq, hk, f = cfg.heads // tp, cfg.kv_heads // tp, cfg.ffn // tp
    out_std = std / math.sqrt(2 * cfg.layers)
    for l in range(cfg.layers):
        s = base + 1000 * (l + 1) + 97 * tp_rank
        wqkv = rnd(((hq + 2 * hk) * D, H), s + 1)
        wo = rnd((H, hq * D), s + 2, out_std)
        if cfg.q_heads_true:       # pad heads: zero Wq rows and Wo columns (exact)
            wqkv[:hq * D].view(hk, cfg.group, D, H)[:, cfg.group_true:] = 0
            wo.view(H, hk, cfg.group, D)[:, :, cfg.group_true:] = 0
        layers.append(LayerWeights(
            attn_norm=norm_w(),
            wqkv=wqkv,
            wo=wo,
            mlp_norm=norm_w(),
            w_gate_up=rnd((2 * f, H), s + 3),
            w_down=rnd((H, f), s + 4, out_std)))
    embed = rnd((cfg.vocab_size, H), base + 11, 1.0)
    return LlamaWeights(embed=embed, layers=layers, final_norm=norm_w(),
                        lm_head=embed if cfg.tie_embeddings else rnd((cfg.vocab_size, H), base + 13))


def fold_norm_weights(w: "LlamaWeights") -> "LlamaWeights":
    """Fold each layer's RMSNorm weights into the projections that consume the
    normed rows (Wqkv <- Wqkv diag(attn_norm), W_gate_up <- W_gate_up
    diag(mlp_norm)) and set the norm weights to ones: the same model, in the
    form the fused-norm forward needs (the GEMM epilogues apply only the
    per-row rsqrt).  In place and idempotent (a second fold multiplies by
    ones), so weights shared by several models, checkpoints written from them
    and reference forwards stay consistent.  Random-init norms are ones
    already (nothing to fold)."""
    for lw in w.layers:
        for norm, name in ((lw.attn_norm, "wqkv"), (lw.mlp_norm, "w_gate_up")):
            if bool((norm == 1).all()):
                continue
            mat = getattr(lw, name)
            g = norm.float()[None, :]
            for r0 in range(0, mat.shape[0], 4096):       # bounded fp32 temporaries
                blk = mat[r0:r0 + 4096]
                blk.copy_((blk.float() * g).to(mat.dtype))
            norm.fill_(1)
    return w


class LlamaModel:
    """Stateless forward over weights + an external paged KV cache."""

    def __init__(self, cfg: LlamaConfig, weights: LlamaWeights, device, tp_rank: int = 0,
                 tp: int = 1, tp_group=None, allreduce=None, seq_parallel: Optional[bool] = None,
                 sp_collectives=None):
        self.cfg = cfg
        self.w = weights
        self.device = torch.device(device)
        self.tp_rank, self.tp, self.tp_group = tp_rank, tp, tp_group
        if cfg.heads % tp or cfg.kv_heads % tp or cfg.ffn % tp:
            raise ValueError(f"tp={tp} does not divide heads/kv_heads/ffn of {cfg.name}")
        if cfg.head_dim != 128 or 16 % cfg.group:
            # attention packs 16 MFMA rows as (16 / group) tokens x group heads of d=128
            raise NotImplementedError(f"{cfg.name}: head_dim {cfg.head_dim} / GQA group {cfg.group} "
                                      "not served by the gfx950 kernels (need d=128, group | 16; "
                                      "models.llama.pad_gqa pads the query heads)")
        self.hq, self.hkv = cfg.heads // tp, cfg.kv_heads // tp
        # RMSNorm fused into the GEMM epilogues (TP = 1, no sequence parallel):
        # residual projections accumulate each row's sum of squares, the
        # consumers scale their accumulators by the row's rsqrt; the norm
        # weights are folded into Wqkv / W_gate_up.  MCP_FUSED_NORM=0: the
        # standalone RMSNorm kernel between the projections.
        fold_norm_weights(self.w)
        self.cos_sin = ref.rope_cos_sin(cfg.max_pos, cfg.head_dim, cfg.rope_theta, self.device,
                                        cfg.rope_scaling)
        self.scale = 1.0 / math.sqrt(cfg.head_dim)
        # weight prefetch: side stream and sink made here, never inside a capture
        self._pf_side = None
        if _PF_ON and self.device.type == "cuda":
            self._pf_side = torch.cuda.Stream(device=self.device)
            ops.weight_prefetch_init(self.device)
        self._allreduce = allreduce      # injectable (simulated ranks in tests)
        if tp > 1 and allreduce is None:
            from ..parallel.comm import make_allreduce
            self._allreduce = make_allreduce(tp_group, self.device)
        # the all-reduces of the row-chunked MLP block (made here, never
        # inside a capture)
        self._comm = None
        self._overlap_min_t = int(os.environ.get("MCP_TP_OVERLAP_MIN_T", str(_TP_OVERLAP_MIN_T)))
        if tp > 1 and self.device.type == "cuda" and self._overlap_min_t > 0:
            self._comm = torch.cuda.Stream(device=self.device)
        if seq_parallel is None:
            seq_parallel = os.environ.get("MCP_SEQ_PARALLEL", "0") == "1"
        self.seq_parallel = bool(seq_parallel) and tp > 1
        # at TP > 1 the statistic comes out of the all-reduce (K12 adds it as
        # it writes the summed rows; RCCL / gloo: a row_sumsq pass after it)
        self.fused_norm = (not self.seq_parallel
                           and os.environ.get("MCP_FUSED_NORM", "1") == "1")
        self._sp = sp_collectives          # (reduce_scatter, all_gather), injectable
        if self.seq_parallel and sp_collectives is None:
            from ..parallel.comm import make_sp_collectives
            self._sp = make_sp_collectives(tp_group, self.device)

    @classmethod
    def random(cls, name: str, device, seed: int = 0, tp_rank: int = 0, tp: int = 1, tp_group=None):
        cfg = get_config(name)
        return cls(cfg, random_weights(cfg, device, seed=seed, tp_rank=tp_rank, tp=tp), device,
                   tp_rank, tp, tp_group)

    def comm_check(self) -> None:
        """Raise if a collective of an earlier step failed (K12 peer timeout)."""
        chk = getattr(self._allreduce, "check", None)
        if chk is not None:
            chk()

    def logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """[R, V] fp32 logits of ``forward``'s rows (free generation, scoring)."""
        return ops.gemm_f32out(hidden, self.w.lm_head)

    # --------------------------------------------------------------- forward
    def _residual_gemm(self, a: torch.Tensor, w: torch.Tensor, x: torch.Tensor) -> torch.Tensor:
        """x + a w^T with the residual add fused in the GEMM epilogue; for TP the
        row-parallel partial sums are all-reduced (rank 0 carries the residual)."""
        if self.tp == 1:
            return ops.gemm(a, w, R=x, out=x)
        y = ops.gemm(a, w, R=x if self.tp_rank == 0 else None)
        self._allreduce(y)
        return y

    @staticmethod
    def _pad_rows(t: torch.Tensor, rows: int) -> torch.Tensor:
        if t.shape[0] == rows:
            return t
        out = t.new_zeros(rows, *t.shape[1:])
        out[:t.shape[0]] = t
        return out

    def _sp_reduce_norm(self, a: torch.Tensor, w: torch.Tensor, x_sh: torch.Tensor,
                        norm_w: torch.Tensor, Tp: int) -> torch.Tensor:
        """Sequence-parallel row-parallel GEMM: partial ``a w^T`` over padded
        rows, reduce-scatter to this rank's rows, then ``x_sh +=`` and RMSNorm
        fused in one kernel.  Returns the normed rows."""
        T = a.shape[0]
        y = torch.empty(Tp * self.tp, w.shape[0], device=a.device, dtype=a.dtype)
        if Tp * self.tp > T:
            y[T:].zero_()
        ops.gemm(a, w, out=y[:T])
        return ops.add_rmsnorm(self._sp[0](y), x_sh, norm_w, self.cfg.eps)

    def forward(self, step, kv) -> torch.Tensor:
        """Runs one ragged step; returns final-normed hidden states of
        ``step.logit_rows`` ([R, H], bf16)."""
        cfg, D = self.cfg, self.cfg.head_dim
        T = step.token_ids.numel()
        x = ops.embedding(step.token_ids, self.w.embed)
        L = cfg.layers
        if self.fused_norm:
            return self._forward_fused_norm(step, kv, x)
        sp = self.seq_parallel
        if sp:
            # x: this rank's Tp rows of the residual stream (T padded to tp*Tp)
            Tp = -(-T // self.tp)
            x = self._pad_rows(x, Tp * self.tp)[self.tp_rank * Tp:(self.tp_rank + 1) * Tp].clone()
            h = self._sp[1](ops.rmsnorm(x, self.w.layers[0].attn_norm, cfg.eps))[:T]
        else:
            h = ops.rmsnorm(x, self.w.layers[0].attn_norm, cfg.eps)
        q = torch.empty(T, self.hq, D, device=h.device, dtype=h.dtype)
        rows = step.logit_rows
        for l in range(L):
            lw = self.w.layers[l]
            kc, vc = kv.layer(l)
            if sp and l + 1 < L:
                ops.qkv_rope(h, lw.wqkv, step.positions, step.slots, self.cos_sin, q, kc, vc,
                             self.hq, self.hkv, D)
                a = ops.paged_attention(q, kc, vc, step.attn, self.scale)
                h = self._sp[1](self._sp_reduce_norm(a.view(T, self.hq * D), lw.wo, x,
                                                     lw.mlp_norm, Tp))[:T]
                act = ops.gemm_silu(h, lw.w_gate_up)
                h = self._sp[1](self._sp_reduce_norm(act, lw.w_down, x,
                                                     self.w.layers[l + 1].attn_norm, Tp))[:T]
                continue
            if sp:
                # last layer: gather the residual once, then the row-selected path
                x = self._sp[1](x)[:T].contiguous()
            # q, K/V cache <- rope(h Wqkv^T): rotation + paged write fused in the
            # GEMM epilogue on the AGPR path (ops.qkv_rope)
            ops.qkv_rope(h, lw.wqkv, step.positions, step.slots, self.cos_sin, q, kc, vc,
                         self.hq, self.hkv, D)
            if l + 1 == L:
                # last layer: every token's K/V is in the cache now, but only the
                # sampled rows' hidden states are read - the output projection
                # and the MLP run on those rows alone (exact; ~1/32 of the
                # O + MLP FLOPs of a step whose tokens are mostly prompt /
                # jump-forward spans)
                if rows.numel() == 0:
                    return x.new_empty(0, cfg.hidden)
                a = ops.paged_attention(q, kc, vc, step.attn, self.scale)
                ri = rows.long()
                x = x.index_select(0, ri)
                a = a.view(T, self.hq * D).index_select(0, ri)
                T = ri.numel()
            else:
                a = ops.paged_attention(q, kc, vc, step.attn, self.scale)
            x = self._residual_gemm(a.view(T, self.hq * D), lw.wo, x)
            h = ops.rmsnorm(x, lw.mlp_norm, cfg.eps)
            act = ops.gemm_silu(h, lw.w_gate_up)          # SwiGLU fused in the epilogue
            x = self._residual_gemm(act, lw.w_down, x)
            if l + 1 < L:
                h = ops.rmsnorm(x, self.w.layers[l + 1].attn_norm, cfg.eps)
        return ops.rmsnorm(x, self.w.final_norm, cfg.eps)

    def _residual_gemm_ss(self, a: torch.Tensor, w: torch.Tensor, x: torch.Tensor,
                          ss_out: torch.Tensor) -> torch.Tensor:
        """x + a w^T with the output rows' fused-norm statistic: in the GEMM
        epilogue at TP = 1; at TP > 1 the row-parallel partials (rank 0 adds
        the residual) are all-reduced and the collective adds the statistic
        (``AllReduce(ss_out=)``; an injected all-reduce without it gets a
        ``row_sumsq`` pass)."""
        if self.tp == 1:
            return ops.gemm(a, w, R=x, out=x, ss_out=ss_out)
        y = ops.gemm(a, w, R=x if self.tp_rank == 0 else None)
        if getattr(self._allreduce, "supports_ss", False):
            self._allreduce(y, ss_out=ss_out)
        else:
            self._allreduce(y)
            ops.row_sumsq(y, ss_out)
        return y

    def _forward_fused_norm(self, step, kv, x) -> torch.Tensor:
        """Forward with every RMSNorm but the final one fused into the
        GEMM epilogues (TP > 1: into the all-reduce) (no normed copy of the residual stream is written):
        ``ss[l, 0]`` / ``ss[l, 1]`` are the fixed-point row sums of squares of
        layer l's attention / MLP input, produced by the previous residual
        GEMM (the embedding: ``row_sumsq``) and consumed by QKV + RoPE /
        SwiGLU, which scale their accumulators per row (norm weights folded
        into their weights, ``fold_norm_weights``)."""
        cfg, D = self.cfg, self.cfg.head_dim
        T = x.shape[0]
        L, eps = cfg.layers, cfg.eps
        rows = step.logit_rows
        # rows: the tokens, or the last layer's selected rows (a hipGraph
        # bucket's row capacity can exceed its token capacity)
        ss = torch.zeros(L + 1, 2, max(T, rows.numel()), dtype=torch.int64, device=x.device)
        ops.row_sumsq(x, ss[0, 0])
        q = torch.empty(T, self.hq, D, device=x.device, dtype=x.dtype)
        side = self._prefetch_stream(x, T)
        for l in range(L):
            lw = self.w.layers[l]
            kc, vc = kv.layer(l)
            ops.qkv_rope(x, lw.wqkv, step.positions, step.slots, self.cos_sin, q, kc, vc,
                         self.hq, self.hkv, D, ss_in=ss[l, 0], eps=eps)
            if side is not None:
                # decode-sized step: while the (latency-bound) attention runs,
                # a second stream reads the o-projection's weights and the head
                # of gate|up once, so those GEMMs stream them from the Infinity
                # Cache (csrc/prefetch.hip); joined after the layer
                cur = torch.cuda.current_stream(x.device)
                side.wait_stream(cur)
                with torch.cuda.stream(side):
                    ops.weight_prefetch(lw.wo, -1, _PF_WGS)
                    rest = _PF_BYTES - lw.wo.numel() * lw.wo.element_size()
                    if rest > 0:
                        ops.weight_prefetch(lw.w_gate_up, rest, _PF_WGS)
            if (self.tp == 1 and l + 1 < L and x.is_cuda and side is None
                    and ops.attention_oproj(q, kc, vc, step.attn, self.scale, lw.wo, x,
                                            ss_out=ss[l, 1])):
                # decode-sized step: attention and the o-projection (+ residual,
                # fused-norm statistic) in one launch, the o weights streaming
                # under the attention's latency chain (csrc/attention_decode.hip)
                act = ops.gemm_silu(x, lw.w_gate_up, ss_in=ss[l, 1], eps=eps)
                x = self._residual_gemm_ss(act, lw.w_down, x, ss[l + 1, 0])
                continue
            a = ops.paged_attention(q, kc, vc, step.attn, self.scale)
            if l + 1 == L:
                # last layer: only the sampled rows go on (see ``forward``)
                if rows.numel() == 0:
                    if side is not None:             # join the prefetch before leaving
                        torch.cuda.current_stream(x.device).wait_stream(side)
                    return x.new_empty(0, cfg.hidden)
                ri = rows.long()
                x = x.index_select(0, ri)
                a = a.view(T, self.hq * D).index_select(0, ri)
                T = ri.numel()
            if self._comm is not None and l + 1 < L and T >= self._overlap_min_t:
                x = self._mlp_block_overlapped(a.view(T, self.hq * D), lw, x, ss[l, 1],
                                               ss[l + 1, 0], eps)
            else:
                x = self._residual_gemm_ss(a.view(T, self.hq * D), lw.wo, x, ss[l, 1])
                act = ops.gemm_silu(x, lw.w_gate_up, ss_in=ss[l, 1], eps=eps)
                x = self._residual_gemm_ss(act, lw.w_down, x, ss[l + 1, 0])
            if side is not None:
                torch.cuda.current_stream(x.device).wait_stream(side)
        return ops.rmsnorm(x, self.w.final_norm, eps)

    def _ar(self, y: torch.Tensor, ss_out: torch.Tensor) -> None:
        """All-reduce of row-parallel partials + the rows' fused-norm statistic."""
        if getattr(self._allreduce, "supports_ss", False):
            self._allreduce(y, ss_out=ss_out)
        else:
            self._allreduce(y)
            ops.row_sumsq(y, ss_out)

    def _mlp_block_overlapped(self, a: torch.Tensor, lw, x: torch.Tensor, ss_mid: torch.Tensor,
                              ss_next: torch.Tensor, eps: float) -> torch.Tensor:
        """TP > 1: o-projection + all-reduce,
        gate|up, down + all-reduce as two row chunks.  Every op of this block is
        row-wise, so chunk c's all-reduce runs on the comm stream while the
        compute stream does the other chunk's GEMMs: AR(o, 0) under o(1),
        AR(o, 1) under gate|up + down of chunk 0, AR(down, 0) under chunk 1's
        MLP; only AR(down, 1) stays exposed.  The arithmetic per row is the
        unchunked block's (each row's sums, the same collective per element)."""
        T = x.shape[0]
        h = min(T - 1, max(64, (T // 2 + 63) // 64 * 64))
        cur = torch.cuda.current_stream(x.device)
        comm = self._comm
        rank0 = self.tp_rank == 0
        y = torch.empty_like(x)
        z = torch.empty_like(x)
        chunks = ((0, h), (h, T))
        done_o = []
        for r0, r1 in chunks:
            ops.gemm(a[r0:r1], lw.wo, R=x[r0:r1] if rank0 else None, out=y[r0:r1])
            comm.wait_stream(cur)
            with torch.cuda.stream(comm):
                self._ar(y[r0:r1], ss_mid[r0:r1])
                done_o.append(comm.record_event())
        done_down = []
        for (r0, r1), ev in zip(chunks, done_o):
            cur.wait_event(ev)
            act = ops.gemm_silu(y[r0:r1], lw.w_gate_up, ss_in=ss_mid[r0:r1], eps=eps)
            ops.gemm(act, lw.w_down, R=y[r0:r1] if rank0 else None, out=z[r0:r1])
            comm.wait_stream(cur)
            with torch.cuda.stream(comm):
                self._ar(z[r0:r1], ss_next[r0:r1])
                done_down.append(comm.record_event())
        for ev in done_down:
            cur.wait_event(ev)
        return z

    def _prefetch_stream(self, x, T):
        """The side stream of the weight prefetch (MCP_WEIGHT_PREFETCH=1) for
        steps of at most _PF_MAX_T tokens, else None."""
        if not (_PF_ON and x.is_cuda and T <= _PF_MAX_T):
            return None
        return self._pf_side
