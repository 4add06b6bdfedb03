"""Plain, slow statement of the Topelorn decoder, one function per mechanism.

Whole sequences, one at a time: no cache, no pages, no batching, no padding, no
absorbed projections, nothing fused.  Weights are a dict of named tensors in the
checkpoint's own layout (``l<i>.mix.q`` and so on), the configuration is the
parsed config.json.  Shares no code with the package; the tests compare the
engine with it.  ``dtype`` picks the arithmetic (float64 by default).
"""
import math

import torch


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def rotate_halves(x, positions, rot):
    """x [T, heads, dim]: dimension i turns with i + dims / 2, the dimensions
    from ``dims`` on stay."""
    n = rot["dims"]
    y = x.clone()
    for i in range(n // 2):
        f = float(rot["base"]) ** (-2 * i / n)
        a = torch.tensor([p * f for p in positions], dtype=torch.float64)
        c, s = a.cos().to(x.dtype)[:, None], a.sin().to(x.dtype)[:, None]
        u, v = x[..., i], x[..., i + n // 2]
        y[..., i] = u * c - v * s
        y[..., i + n // 2] = v * c + u * s
    return y


def window_mask(T, size, keep_first):
    """[T, T] bool: query row i sees key column j."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def slope(head, heads):
    return 2.0 ** (-8.0 * (head + 1) / heads)


def distance_bias(T, head, heads, dtype):
    """[T, T]: what head ``head`` loses per token of distance."""
    i = torch.arange(T, dtype=dtype)[:, None]
    j = torch.arange(T, dtype=dtype)[None, :]
    return slope(head, heads) * (i - j)


def softmax(scores, mask, sink=None):
    """Weights of the visible keys; ``sink``: one more score in the denominator."""
    s = scores.masked_fill(~mask, -math.inf)
    m = s.amax(-1, keepdim=True)
    if sink is not None:
        m = torch.maximum(m, sink)
    e = torch.exp(s - m)
    den = e.sum(-1, keepdim=True)
    if sink is not None:
        den = den + torch.exp(sink - m)
    return e / den


def mix_values(v, first, lam):
    return (1 - lam) * v + lam * first


def head_gate(out, h, wg):
    """out [T, heads, vdim] times one sigmoid per token and head."""
    return out * torch.sigmoid(h @ wg.T)[..., None]


def attention(h, w, pre, m, eps, first):
    """(output, the layer's projected values); ``first``: the first mixed
    layer's values of the same tokens, None where nothing is mixed in."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm((h @ w[pre + "q"].T).view(T, H, d), w[pre + "q.norm"], eps)
    k = rms_norm((h @ w[pre + "k"].T).view(T, G, d), w[pre + "k.norm"], eps)
    v = own = (h @ w[pre + "v"].T).view(T, G, dv)
    if first is not None:
        v = mix_values(own, first, w[pre + "vmix"])
    mask = window_mask(T, m["mask"]["size"], m["mask"].get("keep_first", 0))
    heads = []
    for i in range(H):
        g = i // (H // G)
        s = (q[:, i] @ k[:, g].T) * m["scale"] - distance_bias(T, i, H, h.dtype)
        heads.append(softmax(s, mask, w[pre + "sink"][i]) @ v[:, g])
    out = head_gate(torch.stack(heads, 1), h, w[pre + "g"])
    return out.reshape(T, H * dv) @ w[pre + "o"].T, own


def latent_attention(h, w, pre, m, eps):
    T = h.shape[0]
    H, d, r, dv, n = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ w[pre + "q"].T).view(T, H, d + r)
    down = h @ w[pre + "dkv"].T
    c = rms_norm(down[:, :n], w[pre + "dkv.norm"], eps)
    k_rot = rotate_halves(down[:, None, n:], range(T), m["rot"])[:, 0]
    q_rot = rotate_halves(q[..., d:], range(T), m["rot"])
    k = (c @ w[pre + "uk"].T).view(T, H, d)
    v = (c @ w[pre + "uv"].T).view(T, H, dv)
    mask = window_mask(T, m["mask"]["size"], 0)
    heads = []
    for i in range(H):
        s = (q[:, i, :d] @ k[:, i].T + q_rot[:, i] @ k_rot.T) * m["scale"]
        heads.append(softmax(s, mask) @ v[:, i])
    out = head_gate(torch.stack(heads, 1), h, w[pre + "g"])
    return out.reshape(T, H * dv) @ w[pre + "o"].T


def feed_forward(h, w, pre):
    z = h @ w[pre + "gate"].T
    return (z * torch.sigmoid(z) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def forward(c, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one whole sequence; ``layers_out`` (a list) gets
    the residual stream after every layer."""
    w = {k: t.to(dtype) for k, t in weights.items()}
    eps = c["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)]
    first = None
    for i, ly in enumerate(c["layers"]):
        p, m = f"l{i}.", ly["mixer"]
        h = layer_norm(x, w[p + "norm1"], eps)
        if ly["type"] == "latent_attention":
            y = latent_attention(h, w, p + "mix.", m, eps)
        else:
            mixes = bool(m.get("v_mix"))
            y, own = attention(h, w, p + "mix.", m, eps, first if mixes else None)
            if mixes and first is None:
                first = own
        if ly["mlp"] is not None:
            y = y + feed_forward(h, w, p + "mlp.")
        x = x + y
        if layers_out is not None:
            layers_out.append(x.clone())
    return layer_norm(x, w["final.norm"], eps) @ w["embed"].T
