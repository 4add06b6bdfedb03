"""Plain, slow statement of the Dozazen decoder, one function per mechanism.

Whole sequences, one at a time: no cache, no pages, no batching, no padding,
nothing fused.  Weights are a dict of named tensors in the checkpoint's own
layout (``l<i>.mix.q`` and so on), the configuration is the parsed
config.json.  Shares no code with the package; the tests compare the engine
with it.  ``dtype`` picks the arithmetic (float64 by default).
"""
import math

import torch


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def soft_cap(s, cap):
    return cap * torch.tanh(s / cap)


def frequencies(rot):
    """One rotation frequency per pair of dimensions, long wavelengths slowed."""
    out = []
    sc = rot.get("scaling")
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2 * i / rot["dims"])
        if sc:
            wave = 2 * math.pi / f
            if wave < sc["original"] / sc["high"]:
                pass
            elif wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            else:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate(x, positions, rot):
    """x [T, heads, dim]: neighbouring dimensions (2i, 2i + 1) turn together."""
    y = x.clone()
    for i, f in enumerate(frequencies(rot)):
        a = torch.tensor([p * f for p in positions], dtype=torch.float64)
        c, s = a.cos().to(x.dtype)[:, None], a.sin().to(x.dtype)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i] = u * c - v * s
        y[..., 2 * i + 1] = v * c + u * s
    return y


def chunk_mask(T, size):
    """[T, T] bool: query row i sees key column j."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    return (j <= i) & (i // size == j // size)


def sink_softmax(scores, mask):
    """exp / (1 + sum of exp): one unit of weight goes to no key at all."""
    s = scores.masked_fill(~mask, -math.inf)
    m = s.amax(-1, keepdim=True).clamp(min=0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def attention(h, w, pre, m):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[pre + "q"].T + w[pre + "q.b"]).view(T, H, d)
    k = (h @ w[pre + "k"].T + w[pre + "k.b"]).view(T, G, d)
    v = (h @ w[pre + "v"].T + w[pre + "v.b"]).view(T, G, dv)
    q = rotate(q, range(T), m["rot"])
    k = rotate(k, range(T), m["rot"])
    mask = chunk_mask(T, m["mask"]["size"])
    heads = []
    for i in range(H):
        g = i // (H // G)
        s = soft_cap((q[:, i] @ k[:, g].T) * m["scale"], m["softcap"])
        heads.append(sink_softmax(s, mask) @ v[:, g])
    return torch.cat(heads, -1) @ w[pre + "o"].T


def feed_forward(h, w, pre):
    return (gelu_tanh(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def layer_runs(c):
    """[(layer, starts a pass)] in the order they run."""
    n, lp = len(c["layers"]), c.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    out = [(i, False) for i in range(lp["start"])]
    for _ in range(lp["times"]):
        out += [(i, i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return out + [(i, False) for i in range(lp["stop"], n)]


def forward(c, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one whole sequence; ``layers_out`` (a list) gets
    the residual stream after every layer run."""
    w = {k: t.to(dtype) for k, t in weights.items()}
    eps = c["norm"]["eps"]
    x = x0 = w["embed"][torch.as_tensor(tokens)] * c["embedding"]["scale"]
    for i, begins in layer_runs(c):
        if begins:
            x = torch.cat([x, x0], -1) @ w["loop.in"].T
        ly, p = c["layers"][i], f"l{i}."
        x = x + rms_norm(attention(rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", ly["mixer"]),
                         w[p + "norm1b"], eps)
        if ly["mlp"] is not None:
            x = x + rms_norm(feed_forward(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp."),
                             w[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    z = (rms_norm(x, w["final.norm"], eps) @ w["head"].T) * c["logit_scale"]
    return soft_cap(z, c["logit_softcap"])
