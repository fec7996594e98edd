"""Plain token-by-token oracle of the Gakupel decoder, one function per
mechanism, written for reading and not for speed.

Everything runs in double precision on the CPU from a dict of named tensors
and the configuration dict, for one sequence from position 0, with no cache,
no batching and no code of ``aurora_amd``.
"""

import math

import torch

DT = torch.float64


# ---------------------------------------------------------------- norms, heads

def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def head_norm(x, w, eps):
    """x [T, H, d], each head by itself; w [d] for all of them."""
    return rms(x, eps) * w


def whole_norm(x, w, eps):
    """x [T, H, d], all heads of a token together; w [H * d]."""
    return (rms(x.flatten(1), eps) * w).reshape(x.shape)


def rotate(x, dims, base):
    """x [T, H, d]: dimension i and i + dims/2 turn by p * base^(-2i/dims)."""
    y = x.clone()
    half = dims // 2
    for p in range(x.shape[0]):
        for i in range(half):
            a = p * base ** (-2.0 * i / dims)
            u, v = x[p, :, i], x[p, :, i + half]
            y[p, :, i] = u * math.cos(a) - v * math.sin(a)
            y[p, :, i + half] = v * math.cos(a) + u * math.sin(a)
    return y


def temperature(p, cfg):
    """Factor of the query at position p."""
    return 1 + cfg["coef"] * math.log((p + 1) // cfg["every"] + 1)


def log_distance(r1, r2, dist):
    """What a key ``dist`` tokens back loses."""
    return r1 * torch.log(1 + r2 * dist)


def attend(q, k, v, scale, bias=None, sink=False):
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e], causal. bias(h, dist)
    is taken off the scores; a sink adds one to the softmax's denominator."""
    T, H, _ = q.shape
    group = H // k.shape[1]
    dist = torch.arange(T, dtype=q.dtype).unsqueeze(1) - torch.arange(T, dtype=q.dtype)
    out = []
    for h in range(H):
        s = (q[:, h] @ k[:, h // group].T) * scale
        if bias is not None:
            s = s - bias(h, dist.clamp(min=0))
        s = s.masked_fill(dist < 0, -math.inf)
        top = s.max(-1, keepdim=True).values.clamp(min=0)
        p = torch.exp(s - top)
        whole = p.sum(-1, keepdim=True) + (torch.exp(-top) if sink else 0.0)
        out.append((p / whole) @ v[:, h // group])
    return torch.stack(out, 1)


# --------------------------------------------------------------------- mixers

def attention(h, t, pre, m, eps):
    """Rotary attention with head norms whose values are the keys as projected."""
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = (h @ t[pre + "q"].T).reshape(T, H, d)
    k = (h @ t[pre + "k"].T).reshape(T, G, d)
    v = k
    q = rotate(head_norm(q, t[pre + "q.norm"], eps), m["rot"]["dims"], m["rot"]["base"])
    k = rotate(head_norm(k, t[pre + "k.norm"], eps), m["rot"]["dims"], m["rot"]["base"])
    return attend(q, k, v, m["scale"]).flatten(1) @ t[pre + "o"].T


def biased_attention(h, t, pre, m, eps):
    """Attention without rotation: norms over whole projections, a query
    temperature, a logarithmic distance bias and a sink."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = (h @ t[pre + "q"].T).reshape(T, H, m["dim"])
    k = (h @ t[pre + "k"].T).reshape(T, G, m["dim"])
    v = (h @ t[pre + "v"].T).reshape(T, G, m["vdim"])
    q = whole_norm(q, t[pre + "q.norm"], eps)
    k = whole_norm(k, t[pre + "k.norm"], eps)
    q = torch.stack([q[p] * temperature(p, m["q_temp"]) for p in range(T)])
    r1, r2 = t[pre + "r1"], t[pre + "r2"]
    o = attend(q, k, v, m["scale"], lambda n, dist: log_distance(r1[n], r2[n], dist), True)
    return o.flatten(1) @ t[pre + "o"].T


def short_conv(x, w):
    """Causal convolution per channel and silu; x [T, C], w [C, taps], the last
    column of w multiplies the current token."""
    taps = w.shape[1]
    y = torch.zeros_like(x)
    for i in range(x.shape[0]):
        for j in range(taps):
            src = i - (taps - 1) + j
            if src >= 0:
                y[i] = y[i] + w[:, j] * x[src]
    return silu(y)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, g, beta):
    """q, k [T, H, d], v [T, H, e], g, beta [T, H] -> [T, H, e]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=q.dtype)
    out = torch.zeros_like(v)
    for i in range(T):
        for h in range(H):
            S[h] = g[i, h] * S[h]
            u = beta[i, h] * (v[i, h] - S[h].T @ k[i, h])
            S[h] = S[h] + torch.outer(k[i, h], u)
            out[i, h] = S[h].T @ q[i, h]
    return out


def head_decay(h, t, pre):
    return torch.exp(-torch.exp(t[pre + "A_log"]) * softplus(h @ t[pre + "a"].T + t[pre + "dt_bias"]))


def delta(h, t, pre, m, eps):
    T, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (short_conv(h @ t[pre + n].T, t[pre + n + ".conv"]) for n in "qkv")
    q = (unit(q.reshape(T, G, d)) * d ** -0.5).repeat_interleave(H // G, 1)
    k = unit(k.reshape(T, G, d)).repeat_interleave(H // G, 1)
    beta = torch.sigmoid(h @ t[pre + "b"].T)
    o = delta_rule(q, k, v.reshape(T, H, e), head_decay(h, t, pre), beta)
    o = rms(o, eps) * t[pre + "norm"] * silu(h @ t[pre + "g"].T).reshape(T, H, e)
    return o.flatten(1) @ t[pre + "o"].T


def soft_cap(x, cap):
    return cap * torch.tanh(x / cap)


def matrix_memory(q, k, v, i, f):
    """q, k [T, H, d], v [T, H, e], log gates i, f [T, H] -> [T, H, e]."""
    T, H, d = q.shape
    out = torch.zeros_like(v)
    for h in range(H):
        S = torch.zeros(d, v.shape[2], dtype=q.dtype)
        n = torch.zeros(d, dtype=q.dtype)
        m = torch.zeros((), dtype=q.dtype)
        for t in range(T):
            new = torch.maximum(f[t, h] + m, i[t, h])
            keep, put = torch.exp(f[t, h] + m - new), torch.exp(i[t, h] - new)
            m = new
            S = keep * S + put * torch.outer(k[t, h], v[t, h])
            n = keep * n + put * k[t, h]
            den = torch.maximum((n @ q[t, h]).abs(), torch.exp(-m))
            out[t, h] = (S.T @ q[t, h]) / (den + 1e-6)
    return out


def mlstm(h, t, pre, m, eps):
    T, H, d, e = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ t[pre + "q"].T).reshape(T, H, d) * d ** -0.5
    k = (h @ t[pre + "k"].T).reshape(T, H, d)
    v = (h @ t[pre + "v"].T).reshape(T, H, e)
    i = soft_cap(h @ t[pre + "i"].T + t[pre + "i.b"], m["gate_cap"])
    f = -softplus(-soft_cap(h @ t[pre + "f"].T + t[pre + "f.b"], m["gate_cap"]))
    o = rms(matrix_memory(q, k, v, i, f), eps).flatten(1)
    return (o * t[pre + "norm"] * torch.sigmoid(h @ t[pre + "g"].T)) @ t[pre + "o"].T


def parallel(h, t, pre, m, eps):
    return (m["left_scale"] * biased_attention(h, t, pre + "left.", m["left"], eps)
            + m["right_scale"] * mlstm(h, t, pre + "right.", m["right"], eps))


MIXERS = {"attention": attention, "delta": delta, "parallel": parallel}


# --------------------------------------------------------------- feed-forwards

def softplus(x):
    return torch.log1p(torch.exp(-x.abs())) + x.clamp(min=0)


def silu(x):
    return x * torch.sigmoid(x)


def gelu(x):
    return 0.5 * x * (1 + torch.erf(x / math.sqrt(2)))


def glu(h, t, pre):
    return (silu(h @ t[pre + "gate"].T) * (h @ t[pre + "up"].T)) @ t[pre + "down"].T


def choose(choice, groups, top):
    """Experts of one token: the ``top`` largest choice scores among the groups
    whose two largest add up to most."""
    n = choice.numel() // groups["count"]
    score = [float(c.sort(descending=True).values[:2].sum()) for c in choice.split(n)]
    kept = sorted(range(len(score)), key=lambda g: -score[g])[:groups["keep"]]
    open_ = [e for e in range(choice.numel()) if e // n in kept]
    return sorted(open_, key=lambda e: -float(choice[e]))[:top]


def route(z, correction, router):
    """z [T, E] logits -> dense expert weights [T, E]."""
    s = torch.sigmoid(z)
    out = torch.zeros_like(s)
    for i in range(z.shape[0]):
        at = choose(s[i] + correction, router["groups"], router["top"])
        out[i, at] = s[i, at] / (s[i, at].sum() + 1e-20) * router["scale"]
    return out


def shared_expert(h, t, pre):
    return torch.sigmoid(h @ t[pre + "shared.sg"].T) * glu(h, t, pre + "shared.")


def feed_forward(h, t, pre, f):
    if f["kind"] == "dense":
        return gelu(h @ t[pre + "up"].T) @ t[pre + "down"].T
    w = route(h @ t[pre + "router"].T, t[pre + "correction"], f["router"])
    y = shared_expert(h, t, pre)
    for e in range(f["router"]["experts"]):
        y = y + w[:, e:e + 1] * glu(h, t, f"{pre}e{e}.")
    return y


# ------------------------------------------------------------------------ model

def depth_average(kept, w):
    return sum(w[j] * x for j, x in enumerate(kept))


def forward(cfg, tensors, tokens):
    """Logits [T, vocab] and the residual stream after every layer."""
    t = {k: v.to(DT) if v.is_floating_point() else v for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]

    def norm(x, name):
        return layer_norm(x, t[name], t[name + ".b"], eps)

    x = t["embed"][torch.tensor(list(tokens))]
    kept, trail = [x], []
    for i, layer in enumerate(cfg["layers"]):
        l = f"l{i}."
        x = x + norm(MIXERS[layer["type"]](x, t, l + "mix.", layer["mixer"], eps), l + "norm1")
        if layer["mlp"] is not None:
            x = x + norm(feed_forward(x, t, l + "mlp.", layer["mlp"]), l + "norm2")
        kept.append(x)
        x = depth_average(kept, t[l + "dwa"])
        trail.append(x)
    return norm(x, "final.norm") @ t["head"].T, trail
