"""Plain-PyTorch fp32 reference implementations of every hot op.

These are the numerics oracle for the HIP kernels (tests compare the gfx950
kernels against these at fp32) and the CPU execution path for the engine
(so the whole pipeline runs and is testable without a GPU).

Shapes use the packed-varlen convention throughout:
  * prefill: tokens of all scheduled sequences concatenated on dim 0,
    delimited by ``cu_seqlens`` (int32, [num_seqs+1]).
  * decode: one token per sequence, batch on dim 0.

KV cache layout (chosen for the MI355X decode kernel's streaming reads):
  k_cache, v_cache: [num_pages, n_kv_heads, page_size, head_dim]
  slot = page_id * page_size + offset_in_page
"""
from __future__ import annotations

import math
from typing import Optional, Tuple

import torch


def rmsnorm(x: torch.Tensor, weight: torch.Tensor, eps: float = 1e-5) -> torch.Tensor:
    xf = x.float()
    var = xf.pow(2).mean(-1, keepdim=True)
    y = xf * torch.rsqrt(var + eps) * weight.float()
    return y.to(x.dtype)


def rmsnorm_residual(
    x: torch.Tensor, residual: torch.Tensor, weight: torch.Tensor, eps: float = 1e-5
) -> Tuple[torch.Tensor, torch.Tensor]:
    """Fused residual-add + RMSNorm: returns (normed, new_residual)."""
    new_res = (x.float() + residual.float()).to(x.dtype)
    return rmsnorm(new_res, weight, eps), new_res


def rope_cos_sin_cache(
    head_dim: int, max_pos: int, theta: float = 500000.0, device=None, dtype=torch.float32
) -> torch.Tensor:
    """[max_pos, head_dim] cache: first half cos, second half sin (NeoX/llama pairing:
    dims rotate as (i, i + head_dim//2))."""
    half = head_dim // 2
    inv_freq = 1.0 / (theta ** (torch.arange(0, half, device=device, dtype=torch.float64) / half))
    t = torch.arange(max_pos, device=device, dtype=torch.float64)
    freqs = torch.outer(t, inv_freq)  # [max_pos, half]
    cache = torch.cat([freqs.cos(), freqs.sin()], dim=-1).to(dtype)
    return cache


def rotation_table(dims: int, max_pos: int, base: float, yarn=None) -> torch.Tensor:
    """[max_pos, dims] fp32: the cosines, then the sines of every pair's angle. With
    ``yarn`` (factor, original, fast, slow) the slow pairs turn ``factor`` times slower,
    those between the two limits in part, and all entries grow by 0.1 ln(factor) + 1."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    freq = base ** (-2.0 * i / dims)
    grow = 1.0
    if yarn is not None:
        lo, hi = (dims * math.log(yarn.original / (2 * math.pi * t)) / (2 * math.log(base))
                  for t in (yarn.fast, yarn.slow))
        lo, hi = max(math.floor(lo), 0), min(math.ceil(hi), dims - 1)
        ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0, 1)
        freq = freq / yarn.factor * ramp + freq * (1 - ramp)
        grow += 0.1 * math.log(yarn.factor)
    a = torch.outer(torch.arange(max_pos, dtype=torch.float64), freq)
    return (torch.cat([a.cos(), a.sin()], -1) * grow).float()


def rotate_pairs(x, cos_sin, back: bool = False):
    """x [T, H, d] fp32, cos_sin [T, n]: the first n dimensions turn in neighbouring
    pairs, or ``back``."""
    n = cos_sin.shape[1]
    c, s = cos_sin[:, None, :n // 2], cos_sin[:, None, n // 2:]
    if back:
        s = -s
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    y = x.clone()
    y[..., 0:n:2], y[..., 1:n:2] = u * c - v * s, v * c + u * s
    return y


def rope_apply(
    q: torch.Tensor,  # [T, n_heads, head_dim]
    k: torch.Tensor,  # [T, n_kv_heads, head_dim]
    positions: torch.Tensor,  # [T] int32/int64
    cos_sin: torch.Tensor,  # [max_pos, head_dim]
) -> Tuple[torch.Tensor, torch.Tensor]:
    half = q.shape[-1] // 2
    cs = cos_sin[positions.long()]  # [T, head_dim]
    cos = cs[:, :half].unsqueeze(1).float()  # [T, 1, half]
    sin = cs[:, half:].unsqueeze(1).float()

    def rot(x: torch.Tensor) -> torch.Tensor:
        xf = x.float()
        x1, x2 = xf[..., :half], xf[..., half:]
        return torch.cat([x1 * cos - x2 * sin, x2 * cos + x1 * sin], dim=-1).to(x.dtype)

    return rot(q), rot(k)


def silu_mul(gate_up: torch.Tensor) -> torch.Tensor:
    """[T, 2*I] -> [T, I]: silu(gate) * up, with gate = first half."""
    i = gate_up.shape[-1] // 2
    g = gate_up[..., :i].float()
    u = gate_up[..., i:].float()
    return (g * torch.sigmoid(g) * u).to(gate_up.dtype)


def attention_prefill(
    q: torch.Tensor,  # [T, n_heads, head_dim]
    k: torch.Tensor,  # [T, n_kv_heads, head_dim]
    v: torch.Tensor,  # [T, n_kv_heads, head_dim]
    cu_seqlens: torch.Tensor,  # [num_seqs+1] int32
    scale: float,
    causal: bool = True,
) -> torch.Tensor:
    """Varlen causal attention over freshly-projected K/V (self-contained prefill,
    no cache read). GQA: q heads map to kv head h // (Hq // Hkv)."""
    T, Hq, D = q.shape
    Hkv = k.shape[1]
    g = Hq // Hkv
    out = torch.empty_like(q)
    for s in range(cu_seqlens.numel() - 1):
        a, b = int(cu_seqlens[s]), int(cu_seqlens[s + 1])
        L = b - a
        qs = q[a:b].float()  # [L, Hq, D]
        ks = k[a:b].float().repeat_interleave(g, dim=1)  # [L, Hq, D]
        vs = v[a:b].float().repeat_interleave(g, dim=1)
        att = torch.einsum("qhd,khd->hqk", qs, ks) * scale
        if causal:
            mask = torch.triu(torch.ones(L, L, dtype=torch.bool, device=q.device), diagonal=1)
            att.masked_fill_(mask, float("-inf"))
        p = att.softmax(-1)
        o = torch.einsum("hqk,khd->qhd", p, vs)
        out[a:b] = o.to(q.dtype)
    return out


def attention_prefill_paged(
    q: torch.Tensor,  # [T, n_heads, head_dim] new-chunk queries (packed varlen)
    k_cache: torch.Tensor,  # [num_pages, n_kv_heads, page_size, head_dim]
    v_cache: torch.Tensor,
    block_tables: torch.Tensor,  # [num_seqs, max_pages] int32
    cu_seqlens_q: torch.Tensor,  # [num_seqs+1] int32 (query-chunk lengths)
    context_lens: torch.Tensor,  # [num_seqs] int32: total K len incl. the new chunk
    scale: float,
) -> torch.Tensor:
    """Causal attention of a new query chunk against the paged KV cache.

    The new chunk's K/V must already be written to the cache (kv_cache_write).
    Query i (local index within its chunk) has absolute position
    ctx_len - q_len + i and attends to cache slots [0, pos].  Covers both
    fresh prefill (q_len == ctx_len) and append-prefill of a later agent turn
    (q_len < ctx_len) with one op.
    """
    T, Hq, D = q.shape
    Hkv = k_cache.shape[1]
    g = Hq // Hkv
    P = k_cache.shape[2]
    out = torch.empty_like(q)
    for s in range(cu_seqlens_q.numel() - 1):
        a, b = int(cu_seqlens_q[s]), int(cu_seqlens_q[s + 1])
        qlen = b - a
        L = int(context_lens[s])
        npages = (L + P - 1) // P
        pages = block_tables[s, :npages].long()
        ks = k_cache[pages].permute(1, 0, 2, 3).reshape(Hkv, npages * P, D)[:, :L].float()
        vs = v_cache[pages].permute(1, 0, 2, 3).reshape(Hkv, npages * P, D)[:, :L].float()
        qs = q[a:b].float()  # [qlen, Hq, D]
        att = torch.einsum("qhd,hkd->hqk", qs, ks.repeat_interleave(g, dim=0)) * scale
        # causal: query local i (abs pos L - qlen + i) sees keys <= its abs pos
        kpos = torch.arange(L, device=q.device)
        qpos = torch.arange(L - qlen, L, device=q.device)
        mask = kpos.unsqueeze(0) > qpos.unsqueeze(1)  # [qlen, L]
        att.masked_fill_(mask.unsqueeze(0), float("-inf"))
        p = att.softmax(-1)
        o = torch.einsum("hqk,hkd->qhd", p, vs.repeat_interleave(g, dim=0))
        out[a:b] = o.to(q.dtype)
    return out


def kv_cache_write(
    k: torch.Tensor,  # [T, n_kv_heads, head_dim]
    v: torch.Tensor,
    k_cache: torch.Tensor,  # [num_pages, n_kv_heads, page_size, head_dim]
    v_cache: torch.Tensor,
    slot_mapping: torch.Tensor,  # [T] int32 (page*page_size + offset); -1 = skip
) -> None:
    page_size = k_cache.shape[2]
    valid = slot_mapping >= 0
    slots = slot_mapping[valid].long()
    pages = slots // page_size
    offs = slots % page_size
    k_cache[pages, :, offs] = k[valid].to(k_cache.dtype)
    v_cache[pages, :, offs] = v[valid].to(v_cache.dtype)


def paged_attention_decode(
    q: torch.Tensor,  # [B, n_heads, head_dim] (one new token per seq)
    k_cache: torch.Tensor,  # [num_pages, n_kv_heads, page_size, head_dim]
    v_cache: torch.Tensor,
    block_tables: torch.Tensor,  # [B, max_pages_per_seq] int32
    context_lens: torch.Tensor,  # [B] int32 (total tokens incl. the new one)
    scale: float,
) -> torch.Tensor:
    B, Hq, D = q.shape
    Hkv = k_cache.shape[1]
    g = Hq // Hkv
    P = k_cache.shape[2]
    out = torch.empty_like(q)
    for b in range(B):
        L = int(context_lens[b])
        npages = (L + P - 1) // P
        pages = block_tables[b, :npages].long()
        ks = k_cache[pages].permute(1, 0, 2, 3).reshape(Hkv, npages * P, D)[:, :L].float()
        vs = v_cache[pages].permute(1, 0, 2, 3).reshape(Hkv, npages * P, D)[:, :L].float()
        qs = q[b].float()  # [Hq, D]
        att = torch.einsum("hd,hkd->hk", qs, ks.repeat_interleave(g, dim=0)) * scale
        p = att.softmax(-1)
        o = torch.einsum("hk,hkd->hd", p, vs.repeat_interleave(g, dim=0))
        out[b] = o.to(q.dtype)
    return out


def embed_pool(
    hidden: torch.Tensor,  # [T, H]
    cu_seqlens: torch.Tensor,  # [num_seqs+1]
) -> torch.Tensor:
    """Mean-pool per sequence + L2 normalize (BGE/MiniLM-style sentence embedding)."""
    outs = []
    for s in range(cu_seqlens.numel() - 1):
        a, b = int(cu_seqlens[s]), int(cu_seqlens[s + 1])
        m = hidden[a:b].float().mean(0)
        outs.append(m / (m.norm() + 1e-12))
    return torch.stack(outs).to(hidden.dtype)


def knn_topk(
    query: torch.Tensor,  # [Q, D] (normalized)
    docs: torch.Tensor,  # [N, D] (normalized)
    k: int,
) -> Tuple[torch.Tensor, torch.Tensor]:
    """Brute-force cosine/IP top-k over an HBM-resident doc matrix."""
    scores = query.float() @ docs.float().t()  # [Q, N]
    k = min(k, docs.shape[0])
    vals, idx = scores.topk(k, dim=-1)
    return vals, idx


def softmax_sample(
    logits: torch.Tensor,  # [B, V] float
    temperature: torch.Tensor,  # [B] (0 => greedy)
    top_p: torch.Tensor,  # [B] in (0, 1]
    top_k: torch.Tensor,  # [B] int (0 => off)
    generator: Optional[torch.Generator] = None,
) -> torch.Tensor:
    """Per-row temperature + top-k + top-p sampling; rows with temperature==0 take argmax."""
    B, V = logits.shape
    out = torch.empty(B, dtype=torch.long, device=logits.device)
    lf = logits.float()
    for b in range(B):
        t = float(temperature[b])
        row = lf[b]
        if t <= 0.0:
            out[b] = row.argmax()
            continue
        row = row / t
        tk = int(top_k[b])
        if tk > 0 and tk < V:
            kth = row.topk(tk).values[-1]
            row = row.masked_fill(row < kth, float("-inf"))
        tp = float(top_p[b])
        if tp < 1.0:
            sorted_row, sorted_idx = row.sort(descending=True)
            probs = sorted_row.softmax(-1)
            cum = probs.cumsum(-1)
            cut = cum - probs >= tp  # tokens strictly after the nucleus
            sorted_row = sorted_row.masked_fill(cut, float("-inf"))
            row = torch.full_like(row, float("-inf")).scatter(0, sorted_idx, sorted_row)
        p = row.softmax(-1)
        out[b] = torch.multinomial(p, 1, generator=generator)[0]
    return out


# ---- layer-listed decoders: biased attention, recurrences, routed GLU --------

def residual_rmsnorm(x, weight, eps, delta=None, moe=None, step=None,
                     offset: float = 1.0, dtype=None, gate=None, post=None):
    """x (fp32, updated in place) += delta (times the sigmoid of ``gate`` =
    (pre-activation, bias), if given) and the routed experts' weighted sum, with
    ``post`` both together normed and times it, then += step; returns rms(x) *
    (offset + weight) in ``dtype``."""
    r = torch.zeros_like(x)
    if delta is not None:
        y = delta.float()
        r += y if gate is None else y * torch.sigmoid(gate[0].float() + gate[1])
    if moe is not None:
        y, place, weights = moe
        r += (y.float()[place.long()] * weights.unsqueeze(-1)).sum(1)
    if post is not None:
        r *= torch.rsqrt(r.pow(2).mean(-1, keepdim=True) + eps) * post
    x += r
    if step is not None:
        x += step.float()
    inv = torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)
    return (x * inv * (offset + weight.float())).to(dtype or x.dtype)


def bias_kv_write(proj, cols, bias, slots, k_cache, v_cache,
                  heads: int, kv_heads: int, dim: int, vdim: int):
    """Columns of a fused projection + bias -> q [T, heads, DK] and the paged
    cache; the cache's head widths may exceed dim / vdim (zero filled)."""
    T = proj.shape[0]
    nq, nk, nv = heads * dim, kv_heads * dim, kv_heads * vdim

    def take(c0, b0, n, h, d, width):
        y = proj[:, c0:c0 + n].float() + bias[b0:b0 + n]
        y = y.reshape(T, h, d).to(proj.dtype)
        return torch.nn.functional.pad(y, (0, width - d))

    DK, DV = k_cache.shape[3], v_cache.shape[3]
    q = take(cols[0], 0, nq, heads, dim, DK)
    k = take(cols[1], nq, nk, kv_heads, dim, DK)
    v = take(cols[2], nq + nk, nv, kv_heads, vdim, DV)
    kv_cache_write(k, v, k_cache, v_cache, slots)
    return q


def _paged_rows(cache, pages, L):
    H, P, D = cache.shape[1:]
    return cache[pages].permute(1, 0, 2, 3).reshape(H, -1, D)[:, :L].float()


def biased_attention_paged(q, k_cache, v_cache, block_tables, cu_seqlens_q,
                           context_lens, scale, window, slopes, out, col, vdim,
                           out_scale, log_rate=None, sink=None, chunk=0, turn=None,
                           gate=None):
    """Causal paged attention with a window and a distance penalty slope_h *
    (i - j), or with ``log_rate`` slope_h * ln(1 + rate_h (i - j)), and with
    ``sink`` one more term e^sink_h of the denominator; with ``chunk`` only keys of
    the query's chunk of positions are seen. ``turn`` [positions, vdim] rotates every
    head's result back by the query's position, ``gate`` [T, heads * vdim] multiplies
    it by a sigmoid; writes out[:, col : col + heads * vdim] times out_scale. Decode
    is the case of one query per sequence."""
    T, Hq, _ = q.shape
    P = k_cache.shape[2]
    g = Hq // k_cache.shape[1]
    for s in range(cu_seqlens_q.numel() - 1):
        a, b = int(cu_seqlens_q[s]), int(cu_seqlens_q[s + 1])
        if a == b:
            continue
        L = int(context_lens[s])
        pages = block_tables[s, :(L + P - 1) // P].long()
        ks = _paged_rows(k_cache, pages, L).repeat_interleave(g, 0)
        vs = _paged_rows(v_cache, pages, L).repeat_interleave(g, 0)[..., :vdim]
        att = torch.einsum("qhd,hkd->hqk", q[a:b].float(), ks) * scale
        at = torch.arange(L - (b - a), L, device=q.device).unsqueeze(1)
        keys = torch.arange(L, device=q.device).unsqueeze(0)
        dist = at - keys
        if slopes is not None:
            far = dist.clamp(min=0) if log_rate is None else \
                torch.log(1 + log_rate.view(-1, 1, 1) * dist.clamp(min=0))
            att = att - slopes.view(-1, 1, 1) * far
        hidden = dist < 0
        if window:
            hidden = hidden | (dist >= window)
        if chunk:
            hidden = hidden | (at // chunk != keys // chunk)
        att.masked_fill_(hidden, float("-inf"))
        if sink is not None:
            att = torch.cat([att, sink.view(-1, 1, 1).expand(Hq, b - a, 1)], -1)
        o = torch.einsum("hqk,hkd->qhd", att.softmax(-1)[..., :L], vs) * out_scale
        if turn is not None:
            o = rotate_pairs(o, turn[L - (b - a):L], back=True)
        o = o.reshape(b - a, -1)
        if gate is not None:
            o = o * torch.sigmoid(gate[a:b].float())
        out[a:b, col:col + Hq * vdim] = o.to(out.dtype)


def _l2_unit(x):
    return x * torch.rsqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


def _head_rms(o, eps):
    return o * torch.rsqrt(o.pow(2).mean(-1, keepdim=True) + eps)


def _delta_run(x, z, beta_in, p, start, S, conv):
    """One sequence's tokens from position ``start``: x [n, C] raw q|k|v
    projections, z [n, H*d | H] the decay's pre-activations, S [H, d, e] and conv
    [taps, C] updated in place -> o / rms(o) times the norm's weight."""
    n = x.shape[0]
    H, G, d, e, taps = p.heads, p.kv_heads, p.dim, p.vdim, p.taps
    past = torch.zeros(taps - 1, x.shape[1])
    for j in range(1, taps):
        if start - j >= 0:
            past[taps - 1 - j] = conv[(start - j) % taps].float()
    full = torch.cat([past, x.float()])
    for t in range(max(0, n - taps), n):
        conv[(start + t) % taps] = x[t].to(conv.dtype)
    y = sum(full[j:j + n] * p.conv_w[:, j] for j in range(taps))
    y = y * torch.sigmoid(y)
    q = _l2_unit(y[:, :G * d].reshape(n, G, d)) * d ** -0.5
    k = _l2_unit(y[:, G * d:2 * G * d].reshape(n, G, d))
    v = y[:, 2 * G * d:].reshape(n, H, e)
    q, k = (t.repeat_interleave(H // G, 1) for t in (q, k))
    u = (z.float() + p.dt_bias).reshape(n, H, -1)
    decay = torch.exp(-p.a_log.exp().view(1, H, 1) * torch.nn.functional.softplus(u))
    beta = torch.sigmoid(beta_in.float())
    if start == 0:
        S.zero_()
    o = torch.empty(n, H, e)
    for t in range(n):
        S.mul_(decay[t].unsqueeze(-1))
        w = beta[t].unsqueeze(-1) * (v[t] - torch.einsum("hde,hd->he", S, k[t]))
        S.add_(k[t].unsqueeze(-1) * w.unsqueeze(1))
        o[t] = torch.einsum("hde,hd->he", S, q[t])
    return (_head_rms(o, p.eps) * p.norm).reshape(n, H * e)


def delta_rule(proj, z, p, state, conv, cu, starts, slots, out, col, out_scale):
    """Gated delta rule over packed sequences; slot < 0 rows are skipped."""
    G, d = p.kv_heads, p.dim
    for s in range(len(slots)):
        a, b, slot = int(cu[s]), int(cu[s + 1]), int(slots[s])
        if slot < 0 or a == b:
            continue
        r = proj[a:b]
        x = torch.cat([r[:, p.q0:p.q0 + G * d], r[:, p.k0:p.k0 + G * d],
                       r[:, p.v0:p.v0 + p.heads * p.vdim]], 1)
        nd = p.heads * d
        y = _delta_run(x, z[a:b, :nd], r[:, p.b0:p.b0 + p.heads], p, int(starts[s]),
                       state[slot], conv[slot]) * torch.sigmoid(z[a:b, nd:].float())
        out[a:b, col:col + p.heads * p.vdim] = (y * out_scale).to(out.dtype)


def head_delta_rule(proj, p, state, conv, cu, starts, slots, out, col, out_scale):
    """The rule with one decay per head and a silu gate, all from columns of the
    projection."""
    G, d, H, e = p.kv_heads, p.dim, p.heads, p.vdim
    for s in range(len(slots)):
        a, b, slot = int(cu[s]), int(cu[s + 1]), int(slots[s])
        if slot < 0 or a == b:
            continue
        r = proj[a:b]
        x = torch.cat([r[:, p.q0:p.q0 + G * d], r[:, p.k0:p.k0 + G * d],
                       r[:, p.v0:p.v0 + H * e]], 1)
        y = _delta_run(x, r[:, p.a0:p.a0 + H], r[:, p.b0:p.b0 + H], p, int(starts[s]),
                       state[slot], conv[slot])
        g = r[:, p.g0:p.g0 + H * e].float()
        out[a:b, col:col + H * e] = (y * g * torch.sigmoid(g) * out_scale).to(out.dtype)


def matrix_memory(proj, p, state, norm, top, cu, starts, slots, out, col, out_scale):
    """S_t = e^{f + m - m_t} S + e^{i - m_t} k v', n_t alike with k alone, the
    running maximum m_t = max(f + m, i); state [slots, H, d, e], norm [slots, H, d]
    and top [slots, H] hold S, n and m."""
    H, d, e = p.heads, p.dim, p.vdim
    for s in range(len(slots)):
        a, b, slot = int(cu[s]), int(cu[s + 1]), int(slots[s])
        if slot < 0 or a == b:
            continue
        r, n = proj[a:b].float(), b - a
        take = lambda c, w: r[:, c:c + H * w].reshape(n, H, w)  # noqa: E731
        q, k, v = take(p.q0, d) * d ** -0.5, take(p.k0, d), take(p.v0, e)
        i, f = (p.cap * torch.tanh((r[:, c:c + H] + bias) / p.cap)
                for c, bias in ((p.i0, p.i_bias), (p.f0, p.f_bias)))
        f = torch.nn.functional.logsigmoid(f)
        S, N, M = state[slot], norm[slot], top[slot]
        if int(starts[s]) == 0:
            S.zero_(), N.zero_(), M.zero_()
        o = torch.empty(n, H, e)
        for t in range(n):
            new = torch.maximum(f[t] + M, i[t])
            keep, put = torch.exp(f[t] + M - new), torch.exp(i[t] - new)
            M.copy_(new)
            S.mul_(keep.view(H, 1, 1)).add_(torch.einsum("hd,he->hde", k[t] * put.view(H, 1), v[t]))
            N.mul_(keep.view(H, 1)).add_(k[t] * put.view(H, 1))
            den = torch.maximum((N * q[t]).sum(-1).abs(), torch.exp(-M))
            o[t] = torch.einsum("hde,hd->he", S, q[t]) / (den + 1e-6).unsqueeze(-1)
        y = _head_rms(o, p.eps).reshape(n, H * e) * p.norm
        y = y * torch.sigmoid(r[:, p.g0:p.g0 + H * e])
        out[a:b, col:col + H * e] = (y * out_scale).to(out.dtype)


def retention(proj, p, state, cu, starts, slots, out):
    """Fixed-decay linear attention over packed sequences."""
    H, d, e, half = p.heads, p.dim, p.vdim, p.rot_dims // 2
    for s in range(len(slots)):
        a, b, slot, start = int(cu[s]), int(cu[s + 1]), int(slots[s]), int(starts[s])
        if slot < 0 or a == b:
            continue
        n = b - a
        cs = p.cos_sin[start:start + n].unsqueeze(1)
        cos, sin = cs[..., :half], cs[..., half:]

        def rot(c0):
            x = proj[a:b, c0:c0 + H * d].float().reshape(n, H, d)
            u, w = x[..., :half], x[..., half:2 * half]
            return torch.cat([u * cos - w * sin, w * cos + u * sin, x[..., 2 * half:]], -1)

        q, k = rot(p.q0), rot(p.k0) * d ** -0.5
        v = proj[a:b, p.v0:p.v0 + H * e].float().reshape(n, H, e)
        S = state[slot]
        if start == 0:
            S.zero_()
        o = torch.empty(n, H, e)
        for t in range(n):
            S.mul_(p.decay.view(H, 1, 1)).add_(k[t].unsqueeze(-1) * v[t].unsqueeze(1))
            o[t] = torch.einsum("hde,hd->he", S, q[t])
        g = proj[a:b, p.g0:p.g0 + H * e].float()
        out[a:b] = (_head_rms(o, p.eps).reshape(n, -1) * g * torch.sigmoid(g)).to(out.dtype)


def moe_route(h, router, bias, top: int):
    """fp32 logits -> (expert ids [T, top] int32, softmax over the chosen)."""
    z = h.float() @ router.float().t() + bias
    val, sel = z.topk(top, dim=-1)
    return sel.to(torch.int32), val.softmax(-1)


def moe_clamped_glu(h, sel, w_gate_up, w_down, limit: float, alpha: float,
                    shift: float = 1.0):
    """Every chosen expert's output, unweighted: (y [T*top, W], place [T, top])
    with place giving the row of each choice. Without a limit, alpha 1 and shift 0
    make the activation silu(gate) * up."""
    T, top = sel.shape
    ff = w_down.shape[2]
    y = h.new_empty(T * top, h.shape[1])
    flat = sel.reshape(-1).long()
    tok = torch.arange(T * top) // top
    for e in range(w_down.shape[0]):
        rows = (flat == e).nonzero().flatten()
        if rows.numel() == 0:
            continue
        gu = h[tok[rows]].float() @ w_gate_up[e].float().t()
        g = gu[:, :ff].clamp(max=limit)
        u = gu[:, ff:].clamp(-limit, limit)
        a = (g * torch.sigmoid(alpha * g) * (u + shift)).to(h.dtype)
        y[rows] = (a.float() @ w_down[e].float().t()).to(h.dtype)
    return y, torch.arange(T * top, dtype=torch.int32).view(T, top)


# ---- layer-listed decoders: pair embedding, input convolution, latent attention

def embed_pairs(ids, table, scale, pairs, mul_prev, mul_cur, weight, eps, prev,
                cu, starts, slots, out):
    """rms(table[id] * scale + pairs[row]) * weight per token, fp32 into
    ``out``; row = (previous id * mul_prev + id * mul_cur) mod (rows - 1), the
    last row at position 0. prev [slots, 1] holds each sequence's last id and
    is advanced; slot < 0 rows have no past and store nothing."""
    buckets = pairs.shape[0] - 1
    for s in range(cu.numel() - 1):
        a, b, start, slot = int(cu[s]), int(cu[s + 1]), int(starts[s]), int(slots[s])
        if a == b:
            continue
        cur = ids[a:b].long()
        row = torch.full_like(cur, buckets)
        row[1:] = (cur[:-1] * mul_prev + cur[1:] * mul_cur) % buckets
        if start > 0 and slot >= 0:
            row[0] = (prev[slot, 0].long() * mul_prev + cur[0] * mul_cur) % buckets
        x = table[cur].float() * scale + pairs[row].float()
        out[a:b] = x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps) * weight
        if slot >= 0:
            prev[slot, 0] = cur[-1]


def short_conv_add(h, w, ring, cu, starts, slots, out):
    """out = h + causal convolution of h per channel; w [taps, W]. The ring
    [slots, taps - 1, W] holds position p's h at p mod (taps - 1)."""
    taps = w.shape[0]
    past = taps - 1
    for s in range(cu.numel() - 1):
        a, b, start, slot = int(cu[s]), int(cu[s + 1]), int(starts[s]), int(slots[s])
        n = b - a
        if n == 0:
            continue
        full = torch.zeros(past + n, h.shape[1])
        full[past:] = h[a:b].float()
        if slot >= 0:
            for j in range(1, past + 1):
                if start - j >= 0:
                    full[past - j] = ring[slot, (start - j) % past].float()
            for t in range(max(0, n - past), n):
                ring[slot, (start + t) % past] = h[a + t].to(ring.dtype)
        y = full[past:].clone()
        for j in range(taps):
            y += full[j:j + n] * w[j]
        out[a:b] = y.to(out.dtype)


def normed_columns(proj, col, width, weight, eps):
    x = proj[:, col:col + width].float()
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps) * weight


def latent_write(proj, col, rank, weight, eps, slots, cache, at=None, key_col=None,
                 cos_sin=None):
    """Normed latent of every token into the paged cache [pages, 1, P, R], zero
    filled past ``rank``; with ``cos_sin`` [T, n] the rotated columns from key_col on
    from ``at`` on."""
    c = normed_columns(proj, col, rank, weight, eps)
    P, R = cache.shape[2:]
    rows = torch.nn.functional.pad(c, (0, R - rank))
    if cos_sin is not None:
        n = cos_sin.shape[1]
        k = proj[:, None, key_col:key_col + n].float()
        rows[:, at:at + n] = rotate_pairs(k, cos_sin)[:, 0]
    ok = slots >= 0
    to = slots[ok].long()
    cache[to // P, 0, to % P] = rows.to(cache.dtype)[ok]


def latent_attention(q, gate, uk, uv, sink, scale, cache, block_tables, cu, ctx, out,
                     window=0):
    """q [T, H, D + n], gate [T, H] pre-activations or None, uk [H, D, R], uv [H, E, R]:
    causal attention of every head to keys uk c and values uv c of the cached
    latents c, the sink, if any, in the denominator, times sigmoid(gate) -> out [T,
    H*E]. The cache's columns from R on are more dimensions of every head's key; where
    their number is not n, the surplus is zeros."""
    H, D, R = uk.shape
    P = cache.shape[2]
    n = min(q.shape[2] - D, cache.shape[3] - R)
    q = q[..., :D + n]
    for s in range(cu.numel() - 1):
        a, b, L = int(cu[s]), int(cu[s + 1]), int(ctx[s])
        if a == b:
            continue
        c = _paged_rows(cache, block_tables[s, :(L + P - 1) // P].long(), L)[0]
        k = torch.einsum("hdr,kr->hkd", uk.float(), c[:, :R])
        v = torch.einsum("her,kr->hke", uv.float(), c[:, :R])
        k = torch.cat([k, c[:, R:R + n].expand(H, -1, -1)], -1)
        att = torch.einsum("qhd,hkd->hqk", q[a:b].float(), k) * scale
        dist = torch.arange(L - (b - a), L).unsqueeze(1) - torch.arange(L).unsqueeze(0)
        hidden = (dist < 0) | (dist >= window) if window else dist < 0
        att.masked_fill_(hidden, float("-inf"))
        if sink is not None:
            att = torch.cat([att, sink.view(H, 1, 1).expand(H, b - a, 1)], -1)
        o = torch.einsum("hqk,hke->qhe", att.softmax(-1)[..., :L], v)
        if gate is not None:
            o = o * torch.sigmoid(gate[a:b].float()).unsqueeze(-1)
        out[a:b] = o.reshape(b - a, -1).to(out.dtype)


def xielu(z, act):
    """softplus(act[0]) z^2 + z/2 above zero, (1/2 + softplus(act[1]))
    (e^z - 1 - z) + z/2 below."""
    x = z.float()
    p, q = torch.nn.functional.softplus(act.float())
    low = (0.5 + q) * (torch.expm1(x.clamp(max=0)) - x)
    return (torch.where(x > 0, p * x * x, low) + 0.5 * x).to(z.dtype)


# ---- layer-listed decoders: normed attention heads, output norms, grouped routing

def normed_qkv(proj, p, positions, slots, k_cache, v_cache):
    """Columns of a fused projection -> normed, rotated and scaled queries [T,
    heads, DK], and normed, rotated keys and plain values in the paged cache,
    whose head widths may exceed the model's (zero filled)."""
    T = proj.shape[0]
    DK, DV = k_cache.shape[3], v_cache.shape[3]

    def heads(c0, h, w, d, weight):
        x = proj[:, c0:c0 + h * d].float()
        if weight is not None:
            x = (x if p.whole else x.view(T, h, d))
            x = x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + p.eps) * weight
        return x.reshape(T, h, d)

    def place(x, width):
        return torch.nn.functional.pad(x, (0, width - x.shape[2])).to(proj.dtype)

    def rotated(x):
        if p.cos_sin is None:
            return x
        cs = p.cos_sin[positions.long()].unsqueeze(1)
        half = cs.shape[2] // 2
        cos, sin = cs[..., :half], cs[..., half:]
        u, w = x[..., :half], x[..., half:2 * half]
        return torch.cat([u * cos - w * sin, w * cos + u * sin, x[..., 2 * half:]], -1)

    q = rotated(heads(p.q0, p.heads, DK, p.dim, p.q_norm))
    if p.temp is not None:
        coef, every = p.temp
        step = torch.div(positions.long() + 1, every, rounding_mode="floor") + 1
        q = q * (1 + coef * torch.log(step.float())).view(T, 1, 1)
    k = rotated(heads(p.k0, p.kv_heads, DK, p.dim, p.k_norm))
    v = heads(p.v0, p.kv_heads, DV, p.vdim, None)
    kv_cache_write(place(k, DK), place(v, DV), k_cache, v_cache, slots)
    return place(q, DK)


def _layer_norm(x, weight, bias, eps):
    d = x - x.mean(-1, keepdim=True)
    return d * torch.rsqrt(d.pow(2).mean(-1, keepdim=True) + eps) * weight + bias


def output_norm(src, x, weight, bias, eps, delta=None, gate=None, moe=None, depth=None,
                final=None, dtype=None):
    """x = src + layer_norm(r), r the sub-layer's result: ``delta``, times the
    sigmoid of one number per row, ``gate``, if given, and the chosen experts'
    weighted rows. ``depth`` = (kept [n, T, W], coefs [i + 1]): the sum is kept as
    entry i (if there is room), and x becomes the sum of coefs[j] times entry j.
    Returns x in ``dtype``, with ``final`` = (weight, bias) its layer norm."""
    r = torch.zeros_like(src)
    if delta is not None:
        y = delta.float()
        r += y if gate is None else y * torch.sigmoid(gate.float()).unsqueeze(-1)
    if moe is not None:
        y, place, weights = moe
        r += (y.float()[place.long()] * weights.unsqueeze(-1)).sum(1)
    y = src + _layer_norm(r, weight, bias, eps)
    if depth is not None:
        kept, coefs = depth
        i = coefs.numel() - 1
        if i < kept.shape[0]:
            kept[i] = y
        y = coefs[i] * y + torch.einsum("j,jtw->tw", coefs[:i], kept[:i])
    x.copy_(y)
    return (x if final is None else _layer_norm(x, *final, eps)).to(dtype or x.dtype)


def gelu(z):
    """The exact one: z times the normal distribution function."""
    x = z.float()
    return (0.5 * x * (1 + torch.erf(x * 0.5 ** 0.5))).to(z.dtype)


def silu_glu(z, ff):
    """silu(gate) * up; z [T, 2 ff ...]: gate columns, then up columns."""
    g, u = z[:, :ff].float(), z[:, ff:2 * ff].float()
    return (g * torch.sigmoid(g) * u).to(z.dtype)


def moe_route_grouped(h, router, correction, top: int, groups: int, keep: int, scale: float):
    """Sigmoid scores; the ``top`` best corrected ones among the ``keep`` groups
    whose two best corrected scores add up to most. -> (ids [T, top] int32, the
    chosen plain scores' shares of their sum, times scale)."""
    s = torch.sigmoid(h.float() @ router.float().t())
    T, E = s.shape
    choice = s + correction
    per = choice.view(T, groups, E // groups)
    best = per.topk(min(2, E // groups), dim=-1).values.sum(-1).topk(keep, dim=-1).indices
    closed = torch.ones(T, groups, dtype=torch.bool).scatter_(1, best, False)
    choice = per.masked_fill(closed.unsqueeze(-1), float("-inf")).view(T, E)
    sel = choice.topk(top, dim=-1).indices
    w = s.gather(1, sel)
    return sel.to(torch.int32), w / (w.sum(-1, keepdim=True) + 1e-20) * scale


# ---- layer-listed decoders: convolved attention heads, softmax routing, relu^2

def conv_qkv(proj, p, kv_slots, ring, cu, starts, slots, k_cache, v_cache, q):
    """Columns of a fused projection through the causal convolution; then queries and
    keys turn in their first dimensions and values, with ``p.value_turn``, in all;
    queries to q [T, heads, DK], keys and values to the paged cache, zero filled. The
    ring [slots, taps - 1, C] holds position s's projections at s mod (taps - 1)."""
    H, G, d, e = p.heads, p.kv_heads, p.dim, p.vdim
    taps, C = p.conv_w.shape
    past = taps - 1
    for s in range(cu.numel() - 1):
        a, b, start, slot = int(cu[s]), int(cu[s + 1]), int(starts[s]), int(slots[s])
        n = b - a
        if n == 0:
            continue
        x = torch.cat([proj[a:b, c:c + w] for c, w in
                       ((p.q0, H * d), (p.k0, G * d), (p.v0, G * e))], 1)
        full = torch.zeros(past + n, C)
        full[past:] = x.float()
        if slot >= 0:
            for j in range(1, past + 1):
                if start - j >= 0:
                    full[past - j] = ring[slot, (start - j) % past].float()
            for t in range(max(0, n - past), n):
                ring[slot, (start + t) % past] = x[t].to(ring.dtype)
        y = sum(full[j:j + n] * p.conv_w[j] for j in range(taps))
        turn = p.turn[start:start + n]
        yq = rotate_pairs(y[:, :H * d].reshape(n, H, d), turn)
        yk = rotate_pairs(y[:, H * d:(H + G) * d].reshape(n, G, d), turn)
        yv = y[:, (H + G) * d:].reshape(n, G, e)
        if p.value_turn is not None:
            yv = rotate_pairs(yv, p.value_turn[start:start + n])
        place = lambda t, w: torch.nn.functional.pad(  # noqa: E731
            t, (0, w - t.shape[2])).to(proj.dtype)
        q[a:b] = place(yq, q.shape[2])
        kv_cache_write(place(yk, k_cache.shape[3]), place(yv, v_cache.shape[3]), k_cache,
                       v_cache, kv_slots[a:b])


def relu2(z):
    return z.float().clamp(min=0).pow(2).to(z.dtype)


def moe_route_softmax(h, router, top: int, groups: int, keep: int, scale: float):
    """The ``top`` best experts among the ``keep`` groups with the largest scores,
    a softmax over all experts -> (ids [T, top] int32, chosen scores times scale)."""
    z = h.float() @ router.float().t()
    T, E = z.shape
    per = z.view(T, groups, E // groups)
    best = per.amax(-1).topk(keep, dim=-1).indices
    closed = torch.ones(T, groups, dtype=torch.bool).scatter_(1, best, False)
    sel = per.masked_fill(closed.unsqueeze(-1), float("-inf")).view(T, E).topk(top, dim=-1).indices
    return sel.to(torch.int32), z.softmax(-1).gather(1, sel) * scale


def moe_relu2(h, sel, w_up, w_down):
    """Every chosen expert's output, unweighted, as ``moe_clamped_glu`` gives it."""
    T, top = sel.shape
    y = h.new_empty(T * top, h.shape[1])
    flat = sel.reshape(-1).long()
    tok = torch.arange(T * top) // top
    for e in range(w_down.shape[0]):
        rows = (flat == e).nonzero().flatten()
        if rows.numel():
            a = relu2((h[tok[rows]].float() @ w_up[e].float().t())).to(h.dtype)
            y[rows] = (a.float() @ w_down[e].float().t()).to(h.dtype)
    return y, torch.arange(T * top, dtype=torch.int32).view(T, top)
