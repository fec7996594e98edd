"""Plain oracle of the Fezuzen decoder, one function per mechanism, written for
reading and not for speed.

Everything runs in double precision on the CPU from a dict of named tensors
and the configuration dict, for one sequence from position 0, with no cache,
no batching and no code of ``aurora_amd``.
"""

import math

import torch

DT = torch.float64


# ------------------------------------------------------------ norms, convolutions

def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def causal_conv(u, w):
    """u [T, C], w [C, taps]: the last column of w multiplies the current token."""
    taps = w.shape[1]
    y = torch.zeros_like(u)
    for j in range(taps):
        back = taps - 1 - j
        if back < u.shape[0]:
            y[back:] += w[:, j] * u[:u.shape[0] - back]
    return y


def with_past(h, w):
    """What a sublayer reads: its normed input plus the convolution of it."""
    return h + causal_conv(h, w)


# ------------------------------------------------------------------------ rotation

def frequencies(dims, base, scaling=None):
    """Angle per position of every pair, and the factor of cosine and sine."""
    freq = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return freq, 1.0

    def turns_at(t):
        return dims * math.log(scaling["original"] / (2 * math.pi * t)) / (2 * math.log(base))

    lo = max(math.floor(turns_at(scaling["fast"])), 0)
    hi = min(math.ceil(turns_at(scaling["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freq):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / scaling["factor"] * ramp + f * (1 - ramp))
    return out, 0.1 * math.log(scaling["factor"]) + 1


def turn(x, freq, factor, sign=1):
    """x [T, H, d]: the pair (2i, 2i + 1) of token p turns by sign p freq[i]; the
    dimensions after the last pair stay."""
    T = x.shape[0]
    pos = torch.arange(T, dtype=DT).unsqueeze(1)
    a = pos * torch.tensor(freq, dtype=DT) * sign
    c, s = (torch.cos(a) * factor).unsqueeze(1), (torch.sin(a) * factor).unsqueeze(1)
    n = 2 * len(freq)
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    y = x.clone()
    y[..., 0:n:2] = u * c - v * s
    y[..., 1:n:2] = v * c + u * s
    return y


def rotate(x, rot):
    return turn(x, *frequencies(rot["dims"], rot["base"], rot.get("scaling")))


def rotate_values(v, rot):
    """All of a value's dimensions, never with a scaling."""
    return turn(v, *frequencies(v.shape[2], rot["base"]))


def turn_back(o, rot):
    return turn(o, *frequencies(o.shape[2], rot["base"]), sign=-1)


# ----------------------------------------------------------------------- attention

def in_window(i, j, size):
    return (j <= i) & (i - j < size)


def in_chunk(i, j, size):
    return (j <= i) & (i // size == j // size)


def visible(T, mask, rule):
    i, j = torch.arange(T).unsqueeze(1), torch.arange(T).unsqueeze(0)
    return (j <= i) if mask is None else rule(i, j, mask["size"])


def softmax(s):
    p = torch.exp(s - s.max(-1, keepdim=True).values)
    return p / p.sum(-1, keepdim=True)


def softmax_plus_one(s):
    """One more term of the denominator, e^0."""
    top = s.max(-1, keepdim=True).values.clamp(min=0)
    p = torch.exp(s - top)
    return p / (torch.exp(-top) + p.sum(-1, keepdim=True))


def attend(q, k, v, scale, seen, weigh):
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e]."""
    group = q.shape[1] // k.shape[1]
    out = []
    for h in range(q.shape[1]):
        s = (q[:, h] @ k[:, h // group].T) * scale
        out.append(weigh(s.masked_fill(~seen, -math.inf)) @ v[:, h // group])
    return torch.stack(out, 1)


# -------------------------------------------------------------------------- mixers

def latents(u, t, pre, m, eps):
    """What a layer with latents of its own leaves behind: the normed latents and
    the rotated key part that all heads share."""
    z = u @ t[pre + "dkv"].T
    c = rms_norm(z[:, :m["kv_rank"]], t[pre + "dkv.norm"], eps)
    return c, rotate(z[:, None, m["kv_rank"]:], m["rot"])[:, 0]


def latent_attention(u, kept, t, pre, m, eps):
    c, k_rot = kept
    T, H, d, r = u.shape[0], m["heads"], m["dim"], m["rot_dim"]
    cq = rms_norm(u @ t[pre + "dq"].T, t[pre + "dq.norm"], eps)
    q = (cq @ t[pre + "uq"].T).reshape(T, H, d + r)
    q = torch.cat([q[..., :d], rotate(q[..., d:], m["rot"])], -1)
    k = (c @ t[pre + "uk"].T).reshape(T, H, d)
    k = torch.cat([k, k_rot.unsqueeze(1).expand(T, H, r)], -1)
    v = (c @ t[pre + "uv"].T).reshape(T, H, m["vdim"])
    o = attend(q, k, v, m["scale"], visible(T, m.get("mask"), in_window), softmax)
    return o.flatten(1) @ t[pre + "o"].T


def attention(u, t, pre, m):
    T, H, G = u.shape[0], m["heads"], m["kv_heads"]

    def projected(n):
        return causal_conv(u @ t[pre + n].T, t[pre + n + ".conv"])

    q = rotate(projected("q").reshape(T, H, m["dim"]), m["rot"])
    k = rotate(projected("k").reshape(T, G, m["dim"]), m["rot"])
    v = rotate_values(projected("v").reshape(T, G, m["vdim"]), m["rot"])
    o = attend(q, k, v, m["scale"], visible(T, m.get("mask"), in_chunk), softmax_plus_one)
    o = turn_back(o, m["rot"]).flatten(1)
    return (o * torch.sigmoid(u @ t[pre + "g"].T)) @ t[pre + "o"].T


# ------------------------------------------------------------------------- experts

def relu_squared(z):
    return z.clamp(min=0) ** 2


def expert(h, t, pre):
    return relu_squared(h @ t[pre + ".up"].T) @ t[pre + ".down"].T


def group_score(scores):
    return max(scores)


def choose(scores, r):
    """Indices of the chosen experts of one token."""
    E = len(scores)
    groups = r.get("groups") or {"count": 1, "keep": 1}
    n = E // groups["count"]
    best = sorted(range(groups["count"]),
                  key=lambda g: -group_score(scores[g * n:(g + 1) * n]))[:groups["keep"]]
    allowed = [e for e in range(E) if e // n in best]
    return sorted(allowed, key=lambda e: -scores[e])[:r["top"]]


def share(scores, chosen):
    """The weights of the chosen."""
    return [scores[e] for e in chosen]


def experts(h, t, pre, f):
    out = torch.zeros_like(h)
    scores = softmax(h @ t[pre + "router"].T)
    for p in range(h.shape[0]):
        s = scores[p].tolist()
        chosen = choose(s, f["router"])
        for e, w in zip(chosen, share(s, chosen)):
            out[p] += w * expert(h[p], t, f"{pre}e{e}")
    if f.get("shared"):
        out = out + expert(h, t, pre + "shared")
    return out


# --------------------------------------------------------------------------- model

def forward(cfg, tensors, tokens):
    """Logits [T, vocab] and the residual stream after every layer."""
    t = {k: v.to(DT) if v.is_floating_point() else v for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = t["embed"][torch.as_tensor(tokens)]
    trail, kept = [], {}
    for i, layer in enumerate(cfg["layers"]):
        l, m = f"l{i}.", layer["mixer"]
        u = with_past(rms_norm(x, t[l + "norm1"], eps), t[l + "canon1"])
        if layer["type"] == "latent_attention":
            if m.get("kv_from") is None:
                kept[i] = latents(u, t, l + "mix.", m, eps)
            src = i if m.get("kv_from") is None else m["kv_from"]
            y = latent_attention(u, kept[src], t, l + "mix.", m, eps)
        else:
            y = attention(u, t, l + "mix.", m)
        x = x + rms_norm(y, t[l + "norm1b"], eps)
        if layer["mlp"] is not None:
            u = with_past(rms_norm(x, t[l + "norm2"], eps), t[l + "canon2"])
            x = x + rms_norm(experts(u, t, l + "mlp.", layer["mlp"]), t[l + "norm2b"], eps)
        trail.append(x.clone())
    return rms_norm(x, t["final.norm"], eps) @ t["head"].T * cfg["logit_scale"], trail
