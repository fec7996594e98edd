"""Plain token-by-token oracle of the Senotar decoder, one function per
mechanism, written for reading and not for speed.

Everything runs in double precision on the CPU from a dict of named tensors
and the configuration dict, for one sequence from position 0, with no cache,
no batching and no code of ``aurora_amd``.
"""

import math

import torch

DT = torch.float64


def weighted_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def bigram_row(prev, tok, cfg):
    """Table row of a token and the one before it (None: nothing before)."""
    if prev is None:
        return cfg["buckets"]
    return (prev * cfg["mul_prev"] + tok * cfg["mul_cur"]) % cfg["buckets"]


def embed_tokens(tokens, t, cfg):
    emb = cfg["embedding"]
    rows = []
    for i, tok in enumerate(tokens):
        prev = tokens[i - 1] if i > 0 else None
        rows.append(t["embed"][tok] * emb["scale"] + t["bigram"][bigram_row(prev, tok, emb["bigram"])])
    return weighted_norm(torch.stack(rows), t["embed.norm"], cfg["norm"]["eps"])


def add_short_conv(h, w):
    """h [T, C] plus its causal convolution, w [C, taps]; the last column of w
    multiplies the current token."""
    taps = w.shape[1]
    y = h.clone()
    for i in range(h.shape[0]):
        for j in range(taps):
            src = i - (taps - 1) + j
            if src >= 0:
                y[i] = y[i] + w[:, j] * h[src]
    return y


def sink_attention(q, k, v, sink, scale):
    """q, k [T, H, d], v [T, H, e] -> [T, H, e]: causal; the denominator has
    one more term, e^sink of the head."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        for i in range(T):
            s = (k[:i + 1, h] @ q[i, h]) * scale
            top = max(float(s.max()), float(sink[h]))
            p = torch.exp(s - top)
            out[i, h] = (p / (p.sum() + math.exp(float(sink[h]) - top))) @ v[:i + 1, h]
    return out


def latents(u, t, pre, eps):
    return weighted_norm(u @ t[pre + "dkv"].T, t[pre + "dkv.norm"], eps)


def latent_attention(u, c, t, pre, cfg):
    """u [T, W] the mixer's input, c [T, R] the latents it attends to."""
    T = u.shape[0]
    H, d, e = cfg["heads"], cfg["dim"], cfg["vdim"]
    q = (u @ t[pre + "q"].T).reshape(T, H, d)
    k = (c @ t[pre + "uk"].T).reshape(T, H, d)
    v = (c @ t[pre + "uv"].T).reshape(T, H, e)
    o = sink_attention(q, k, v, t[pre + "sink"], cfg["scale"])
    o = o * torch.sigmoid(u @ t[pre + "g"].T).unsqueeze(-1)
    return o.reshape(T, H * e) @ t[pre + "o"].T


def softplus(x):
    return torch.log1p(torch.exp(-x.abs())) + x.clamp(min=0)


def xielu(z, p, q):
    above = softplus(p) * z * z + z / 2
    below = (0.5 + softplus(q)) * (torch.expm1(z.clamp(max=0)) - z) + z / 2
    return torch.where(z > 0, above, below)


def feed_forward(h, t, pre):
    return xielu(h @ t[pre + "up"].T, *t[pre + "act"]) @ t[pre + "down"].T


def gate(h, t, name):
    return torch.sigmoid(h @ t[name].T + t[name + ".b"])


def forward(cfg, tensors, tokens):
    """Logits [T, vocab] and the residual stream after every layer."""
    t = {k: v.to(DT) if v.is_floating_point() else v for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = embed_tokens(list(tokens), t, cfg)
    trail, kept = [], {}
    for i, layer in enumerate(cfg["layers"]):
        m = layer["mixer"]
        h = weighted_norm(x, t[f"l{i}.norm1"], eps)
        u = add_short_conv(h, t[f"l{i}.canon1"])
        src = m.get("kv_from")
        if src is None:
            src, kept[i] = i, latents(u, t, f"l{i}.mix.", eps)
        x = x + gate(h, t, f"l{i}.rg1") * latent_attention(u, kept[src], t, f"l{i}.mix.", m)
        if layer["mlp"] is not None:
            h = weighted_norm(x, t[f"l{i}.norm2"], eps)
            x = x + gate(h, t, f"l{i}.rg2") * feed_forward(h, t, f"l{i}.mlp.")
        trail.append(x.clone())
    return weighted_norm(x, t["final.norm"], eps) @ t["head"].T, trail
