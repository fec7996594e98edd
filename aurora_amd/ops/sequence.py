"""Ops of the layer-listed decoders: biased window attention over paged KV,
gated delta rules, retention, matrix memories, routed experts, latent
attention, normed and convolved attention heads, pair embeddings, the
sublayers' input convolution and the residual's norms.

Same dispatch rule as the rest of the package: GPU tensors run the gfx950
kernels (bf16, or float32 throughout) and fail loudly without the extension;
CPU tensors run ``torch_ref``.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple

import torch

from . import torch_ref

#: head widths of the matrix-core attention kernels; the paged cache of a
#: bf16 model on the GPU stores heads at the next of these, zero filled
MATRIX_HEAD_DIMS = (64, 128)
#: latent widths of the matrix-core latent attention kernel
MATRIX_LATENT_WIDTHS = (64, 128, 256, 384, 512)
#: columns of a cached latent row per 64 that hold the shared rotated key
KEY_PART = 64
#: widths of spelled-out latent-attention heads, rotated part included
SPELLED_HEAD_DIMS = (64, 128, 192)
#: widest latent of the kernel that serves float32 and everything else
MAX_LATENT = 1024
#: tokens per chunk of the recurrence kernels
RECURRENCE_CHUNK = 16


def cache_head_dims(dim: int, vdim: int, dtype, device) -> Tuple[int, int]:
    """Widths at which the paged cache stores a head's key and value."""
    if torch.device(device).type == "cpu" or dtype != torch.bfloat16:
        return dim, vdim
    pad = [next((w for w in MATRIX_HEAD_DIMS if w >= d), None) for d in (dim, vdim)]
    return (dim, vdim) if None in pad else (pad[0], pad[1])


@dataclass
class DeltaRuleParams:
    """Sizes, projection columns and fp32 weights of a gated delta rule."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int
    q0: int
    k0: int
    v0: int
    b0: int
    conv_w: torch.Tensor   # [2*kv_heads*dim + heads*vdim, taps]
    a_log: torch.Tensor    # [heads]
    dt_bias: torch.Tensor  # [heads*dim]
    norm: torch.Tensor     # [vdim]
    eps: float


@dataclass
class RetentionParams:
    heads: int
    dim: int
    vdim: int
    rot_dims: int
    q0: int
    k0: int
    v0: int
    g0: int
    decay: torch.Tensor    # [heads] fp32
    cos_sin: torch.Tensor  # [positions, rot_dims] fp32
    eps: float


@dataclass
class HeadDeltaParams:
    """The gated delta rule with one decay per head and a silu gate."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int
    q0: int
    k0: int
    v0: int
    b0: int
    a0: int
    g0: int
    conv_w: torch.Tensor   # [2*kv_heads*dim + heads*vdim, taps]
    a_log: torch.Tensor    # [heads]
    dt_bias: torch.Tensor  # [heads]
    norm: torch.Tensor     # [vdim]
    eps: float


@dataclass
class MatrixMemoryParams:
    heads: int
    dim: int
    vdim: int
    q0: int
    k0: int
    v0: int
    i0: int
    f0: int
    g0: int
    i_bias: torch.Tensor   # [heads]
    f_bias: torch.Tensor   # [heads]
    norm: torch.Tensor     # [heads * vdim]
    cap: float
    eps: float


@dataclass
class NormedHeadsParams:
    """Normed queries and keys of an attention; v0 = k0: values are plain keys."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    q0: int
    k0: int
    v0: int
    q_norm: torch.Tensor   # [dim], or [heads * dim] if ``whole``
    k_norm: torch.Tensor
    whole: bool            # one norm over all heads of a token
    eps: float
    cos_sin: Optional[torch.Tensor] = None  # [positions, rotated dims] fp32
    temp: Optional[Tuple[float, int]] = None


def latent_width(rank: int) -> int:
    """Width at which latents are cached, zero filled."""
    if rank > MAX_LATENT:
        raise ValueError(f"latent of {rank} numbers; at most {MAX_LATENT}")
    return next((w for w in MATRIX_LATENT_WIDTHS if w >= rank), -(-rank // 64) * 64)


def latent_head_width(dim: int) -> int:
    """Width of a latent-attention head's rows in the projections' weights."""
    return next((w for w in MATRIX_HEAD_DIMS if w >= dim), -(-dim // 32) * 32)


def latent_rotary_widths(dim: int, rot: int) -> Tuple[int, int, int]:
    """Widths of a rotary latent-attention head: its unrotated and its rotated part
    in the query rows, and the rotated key's columns in a cached row."""
    d = -(-dim // 32) * 32
    whole = next((w for w in SPELLED_HEAD_DIMS if w >= d + rot), d + -(-rot // 32) * 32)
    return d, whole - d, -(-rot // KEY_PART) * KEY_PART


@dataclass
class LatentParams:
    """Sizes, projection columns and weights of latent attention; all head and
    latent widths are the padded ones."""
    heads: int
    dim: int
    vdim: int
    scale: float
    q0: int
    g0: Optional[int]   # None: no gate
    uk: torch.Tensor    # [heads, dim, R]
    uk_t: torch.Tensor  # [heads, R, dim]
    uv: torch.Tensor    # [heads, vdim, R]
    sink: Optional[torch.Tensor]  # [heads] fp32
    #: width of the rotated part behind a query's ``dim`` columns
    tail: int = 0
    cos_sin: Optional[torch.Tensor] = None  # [positions, rotated dims] fp32
    window: int = 0


@dataclass
class LatentFrontParams:
    """Columns of the input projection and weights of what latent attention does
    first; ``c0`` is None where the latents are another layer's."""
    c0: Optional[int]
    rank: int
    weight: Optional[torch.Tensor]    # [rank]
    eps: float
    k0: int = 0                       # the rotated key part
    key_at: int = 0                   # its place in a cached row
    cos_sin: Optional[torch.Tensor] = None
    q0: int = 0                       # the queries' latent
    q_rank: int = 0                   # 0: none
    q_weight: Optional[torch.Tensor] = None


@dataclass
class ConvHeadsParams:
    """Sizes, projection columns and weights of convolved, rotated attention heads."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    q0: int
    k0: int
    v0: int
    conv_w: torch.Tensor   # [taps, heads*dim + kv_heads*(dim + vdim)], the last the present
    turn: torch.Tensor     # [positions, rotated dims] fp32
    value_turn: Optional[torch.Tensor] = None  # [positions, vdim] fp32


@dataclass
class Segment:
    """One regime of a step: prompt portions (``cu`` given) or single tokens
    (row r is sequence r), with what attention and recurrences need."""
    rows: slice
    block_tables: torch.Tensor
    context_lens: torch.Tensor
    starts: torch.Tensor                # position of each sequence's first row
    state_slots: Optional[torch.Tensor]
    cu: Optional[torch.Tensor] = None
    cu_host: Optional[List[int]] = None
    ctx_host: Optional[List[int]] = None
    _maps: Dict[object, object] = field(default_factory=dict)

    @property
    def decode(self) -> bool:
        return self.cu is None

    def cu_or_rows(self, n: int) -> torch.Tensor:
        if self.cu is not None:
            return self.cu
        return torch.arange(n + 1, dtype=torch.int32, device=self.context_lens.device)

    def block_map(self, rows_per_block: int,
                  chunk: int = 0) -> Tuple[torch.Tensor, torch.Tensor]:
        """(sequence, first row within it) of every block of rows; built once
        per step and shared by all layers. With ``chunk`` the blocks are in the order
        of how many keys of their chunk they see."""
        hit = self._maps.get((rows_per_block, chunk))
        if hit is None:
            blocks = []
            for s, (a, b) in enumerate(zip(self.cu_host, self.cu_host[1:])):
                blocks += [(s, o) for o in range(0, b - a, rows_per_block)]
            if chunk:
                first = [c - (b - a) for a, b, c in
                         zip(self.cu_host, self.cu_host[1:], self.ctx_host)]
                blocks.sort(key=lambda x: (first[x[0]] + x[1]) % chunk)
            t = torch.tensor(blocks, dtype=torch.int32).view(-1, 2).t().contiguous().to(
                self.context_lens.device)
            hit = (t[0], t[1])
            self._maps[rows_per_block, chunk] = hit
        return hit

    def chunk_map(self) -> Tuple[torch.Tensor, torch.Tensor, torch.Tensor]:
        """``block_map`` of the recurrences' chunks and every sequence's first
        chunk among them."""
        seq, off = self.block_map(RECURRENCE_CHUNK)
        hit = self._maps.get("first")
        if hit is None:
            first = [0]
            for a, b in zip(self.cu_host, self.cu_host[1:]):
                first.append(first[-1] + -(-(b - a) // RECURRENCE_CHUNK))
            hit = torch.tensor(first, dtype=torch.int32).to(self.context_lens.device)
            self._maps["first"] = hit
        return seq, off, hit


    def latent_map(self, heads: int):
        """(sequence, first row, rows per block) of the blocks of (token, head)
        rows of latent attention; single tokens need no map."""
        if self.decode:
            return None, None, 16 if heads <= 16 else 32
        hit = self._maps.get(("latent", heads))
        if hit is None:
            seq, off = [], []
            for s in range(len(self.cu_host) - 1):
                n = (self.cu_host[s + 1] - self.cu_host[s]) * heads
                off.extend(range(0, n, 32))
                seq.extend([s] * -(-n // 32))
            t = torch.tensor([seq, off], dtype=torch.int32).to(self.context_lens.device)
            hit = (t[0], t[1], 32)
            self._maps[("latent", heads)] = hit
        return hit

    def first_keys(self, window: int) -> List[int]:
        """First key any row of each portion sees through a window (0: none)."""
        return [max(0, c - (b - a) - window + 1) if window else 0 for a, b, c in
                zip(self.cu_host, self.cu_host[1:], self.ctx_host)]

    def latent_rows(self, cache, window: int = 0):
        """Every visible context token's latent, packed, and the place of sequence
        s's token t among them as a table [s, t] (0 where it is not visible); places
        are found once per step."""
        P = cache.shape[2]
        hit = self._maps.get(("context", window))
        if hit is None:
            dev = cache.device
            table = torch.zeros(len(self.ctx_host), max(self.ctx_host), dtype=torch.int32)
            place, n = [], 0
            for s, (lo, c) in enumerate(zip(self.first_keys(window), self.ctx_host)):
                table[s, lo:c] = torch.arange(n, n + c - lo, dtype=torch.int32)
                n += c - lo
                t = torch.arange(lo, c, device=dev)
                place.append(self.block_tables[s].long()[t // P] * P + t % P)
            hit = (torch.cat(place).to(torch.int32), table.to(dev))
            self._maps["context", window] = hit
        return _hip("gather_latents").gather_latents(cache, hit[0]), hit[1]


def _hip(op: str):
    from . import _require_hip
    return _require_hip(op)


def residual_rmsnorm(x, weight, eps, delta=None, moe=None, step=None,
                     offset: float = 1.0, dtype=None, gate=None, post=None):
    if not x.is_cuda:
        return torch_ref.residual_rmsnorm(x, weight, eps, delta, moe, step, offset,
                                          dtype, gate, post)
    return _residual_rmsnorm(x, weight, eps, delta, moe, step, offset, dtype, gate, post)[0]


def _residual_rmsnorm(x, weight, eps, delta, moe, step, offset, dtype, gate, post,
                      conv=(None, None, None, None)):
    y, place, share = moe if moe is not None else (None, None, None)
    pre, bias = gate if gate is not None else (None, None)
    return _hip("residual_rmsnorm").residual_rmsnorm(
        x, weight, delta, pre, bias, y, place, share, post, step, *conv, float(eps),
        float(offset), dtype == torch.bfloat16)


def residual_rmsnorm_conv(x, weight, eps, conv_w, ring, segments: List[Segment],
                          delta=None, moe=None, step=None, offset: float = 1.0,
                          dtype=None, gate=None, post=None):
    """``residual_rmsnorm`` and ``short_conv_add`` of its result: (h, h + conv).
    A step of single tokens does both in one kernel."""
    if x.is_cuda and len(segments) == 1 and segments[0].decode:
        seg = segments[0]
        return tuple(_residual_rmsnorm(x, weight, eps, delta, moe, step, offset, dtype,
                                       gate, post,
                                       (conv_w, ring, seg.starts, seg.state_slots)))
    h = residual_rmsnorm(x, weight, eps, delta, moe, step, offset, dtype, gate, post)
    u = torch.empty_like(h)
    for seg in segments:
        short_conv_add(h, conv_w, ring, seg, u)
    return h, u


def short_conv_add(h, w, ring, seg: Segment, out):
    hs, os_ = h[seg.rows], out[seg.rows]
    if not h.is_cuda:
        torch_ref.short_conv_add(hs, w, ring, seg.cu_or_rows(hs.shape[0]), seg.starts,
                                 seg.state_slots, os_)
        return
    m = _hip("short_conv_add")
    bseq, boff = (None, None) if seg.decode else seg.block_map(m.short_conv_rows())
    m.short_conv_add(hs, w, ring, seg.cu, bseq, boff, seg.starts, seg.state_slots, os_)


def embed_pairs(ids, table, scale, pairs, mul_prev: int, mul_cur: int, weight, eps,
                prev, segments: List[Segment]):
    """fp32 rows of normed token plus pair embeddings; advances ``prev``."""
    out = torch.empty(ids.shape[0], table.shape[1], dtype=torch.float32, device=ids.device)
    for seg in segments:
        i, o = ids[seg.rows], out[seg.rows]
        if ids.is_cuda:
            _hip("embed_pairs").embed_pairs(
                i, table, float(scale), pairs, mul_prev, mul_cur, weight, float(eps),
                prev, seg.cu, seg.starts, seg.state_slots, o)
        else:
            torch_ref.embed_pairs(i, table, scale, pairs, mul_prev, mul_cur, weight, eps,
                                  prev, seg.cu_or_rows(i.shape[0]), seg.starts,
                                  seg.state_slots, o)
    return out


def latent_write(proj, col: int, rank: int, weight, eps, slots, cache):
    latent_front(proj, LatentFrontParams(col, rank, weight, eps), None, slots, cache)


def latent_front(proj, p: LatentFrontParams, positions, slots, cache):
    """Normed latents and the rotated key part to the cache; returns the queries'
    normed latent [T, q_rank], if there is one."""
    turn = p.cos_sin if p.c0 is not None else None
    if not proj.is_cuda:
        if p.c0 is not None:
            torch_ref.latent_write(
                proj, p.c0, p.rank, p.weight, p.eps, slots, cache, p.key_at, p.k0,
                None if turn is None else turn[positions.long()])
        return torch_ref.normed_columns(proj, p.q0, p.q_rank, p.q_weight, p.eps).to(
            proj.dtype) if p.q_rank else None
    cq = torch.empty(proj.shape[0], p.q_rank, dtype=proj.dtype, device=proj.device) \
        if p.q_rank else None
    _hip("latent_front").latent_front(
        proj, -1 if p.c0 is None else p.c0, p.rank, p.weight, float(p.eps), p.k0, p.key_at,
        turn, positions, slots, cache, p.q0, p.q_weight, cq)
    return cq


def rotate_heads(x, positions, cos_sin, out):
    """Neighbouring pairs of the first dimensions of x [T, H, n] turn by their row's
    position, into out [T, H, w] (may be x), zero filled behind them."""
    if not x.is_cuda:
        n = cos_sin.shape[1]
        y = torch_ref.rotate_pairs(x[..., :n].float(), cos_sin[positions.long()])
        out[..., :n] = y.to(out.dtype)
        out[..., n:] = 0
        return
    _hip("rotate_heads").rotate_heads(x, positions, cos_sin, out)


def head_linear(x, w, gate=None, out=None, turn=None):
    """Per-head product: x [T, H, K] (rows may be strided), w [H, N, K] ->
    [T, H, N], times sigmoid(gate [T, H]) if given. ``turn``: the arguments of a
    ``rotate_heads`` of equally many rows and heads to run in the same launch."""
    T, H, _ = x.shape
    if out is None:
        out = torch.empty(T, H, w.shape[1], dtype=x.dtype, device=x.device)
    if x.dtype == torch.bfloat16:
        _hip("head_linear").head_linear(x, w, gate, out, *(turn or (None,) * 4))
        return out
    y = torch.bmm(x.transpose(0, 1).contiguous(), w.transpose(1, 2).contiguous())
    y = y.transpose(0, 1)
    out.copy_(y if gate is None else y * torch.sigmoid(gate).unsqueeze(-1))
    if turn is not None:
        rotate_heads(*turn)
    return out


#: most numbers of spelled-out keys and values one step may hold
EXPANDED_LIMIT = 1 << 31


def expand_latents(seg: Segment, p: LatentParams, rank: int) -> bool:
    """Whether it is faster to spell out every visible key and value of a prompt
    portion's context than to attend in the latents' own space, where a pair of
    tokens costs 2 rank instead of dim + vdim but a key costs nothing."""
    if seg.decode or p.vdim not in MATRIX_HEAD_DIMS or p.dim + p.tail not in (
            SPELLED_HEAD_DIMS if p.tail else MATRIX_HEAD_DIMS):
        return False
    # the flash kernel comes with sink and gate, or with a rotated part and window
    ends = p.sink is not None and p.g0 is not None
    if not (p.sink is None and p.g0 is None if p.tail else ends and not p.window):
        return False
    width = p.dim + p.vdim
    first = seg.first_keys(p.window)
    keys = sum(seg.ctx_host) - sum(first)
    if keys * p.heads * width > EXPANDED_LIMIT:
        return False
    seen = [(b - a) * (c - (b - a) / 2) for a, b, c in
            zip(seg.cu_host, seg.cu_host[1:], seg.ctx_host)]
    if p.window:
        seen = [min(n, (b - a) * p.window) for n, a, b in
                zip(seen, seg.cu_host, seg.cu_host[1:])]
    pairs = sum(seen)
    rows = seg.cu_host[-1]
    # measured rates in flops per us: the latent kernel and the per-head products
    # around it; library products and the flash kernel, which also takes 0.4 us
    # per key and 10^3 of width at least
    latent = pairs * p.heads * 4 * rank / 6e8 + rows * p.heads * 2 * rank * width / 2e8
    product = keys * p.heads * 2 * rank * width / 6e8
    longest = max(min(c, p.window + 256) if p.window else c for c in seg.ctx_host)
    flash = max(pairs * p.heads * 2 * (width + p.tail) / 3e8, longest * width * 4e-4)
    return product + flash < latent


def latent_attention(proj, p: LatentParams, cache, seg: Segment, out, q=None,
                     positions=None):
    """One segment's rows of latent attention into out [rows, H * vdim]. Queries are
    columns of ``proj``, or all rows' q [T, H, dim + tail], whose tails are still to
    be rotated by ``positions``; they may be overwritten."""
    pr, o = proj[seg.rows], out[seg.rows]
    T, H, R, C = pr.shape[0], p.heads, p.uk.shape[2], cache.shape[3]
    if q is None:
        q = pr[:, p.q0:p.q0 + H * p.dim].unflatten(1, (H, p.dim))
    else:
        q, positions = q[seg.rows], positions[seg.rows]
    gate = None if p.g0 is None else pr[:, p.g0:p.g0 + H]
    plain, tail = q[..., :p.dim], q[..., p.dim:]
    if not proj.is_cuda:
        if p.tail:
            rotate_heads(tail, positions, p.cos_sin, tail)
        torch_ref.latent_attention(q, gate, p.uk, p.uv, p.sink, p.scale, cache,
                                   seg.block_tables, seg.cu_or_rows(T),
                                   seg.context_lens, o, p.window)
        return
    m = _hip("latent_attention")
    matrix = (proj.dtype == torch.bfloat16 and R in MATRIX_LATENT_WIDTHS
              and C - R in (0, KEY_PART))
    if matrix and expand_latents(seg, p, R):
        c, rows = seg.latent_rows(cache, p.window)
        k = torch.nn.functional.linear(c[:, :R], p.uk.flatten(0, 1)).view(-1, H, 1, p.dim)
        v = torch.nn.functional.linear(c[:, :R], p.uv.flatten(0, 1)).view(-1, H, 1, p.vdim)
        bseq, boff = seg.block_map(m.biased_prefill_rows(1))
        if p.tail:
            rotate_heads(tail, positions, p.cos_sin, tail)
            m.tailed_attention_prefill(q, k, v, c[:, R:], rows, seg.cu, seg.context_lens,
                                       bseq, boff, p.scale, p.window, o)
        else:
            m.sink_attention_prefill(q, k, v, rows, seg.cu, seg.context_lens, bseq, boff,
                                     p.scale, p.sink, gate, o)
        return
    qa = torch.empty(T, H, C, dtype=q.dtype, device=q.device)
    head_linear(plain, p.uk_t, out=qa[..., :R],
                turn=(tail, positions, p.cos_sin, qa[..., R:]) if p.tail else None)
    if matrix:
        oc = m.latent_attention(qa, cache, seg.block_tables, seg.cu, seg.context_lens,
                                *seg.latent_map(H), p.scale, p.sink, R, p.window)
    else:
        oc = torch.empty(T, H, R, dtype=q.dtype, device=q.device)
        bseq, boff = (None, None) if seg.decode else seg.block_map(1)
        m.latent_attention_rows(qa, cache, seg.block_tables, seg.cu, seg.context_lens,
                                bseq, boff, p.scale, p.sink, p.window, oc)
    head_linear(oc, p.uv, gate, o.unflatten(1, (H, p.vdim)))


def xielu(z, act):
    """Rows of ``z`` may be strided; act [2]: the two slopes before softplus."""
    if not z.is_cuda:
        return torch_ref.xielu(z, act)
    return _hip("xielu").xielu(z, act)


def bias_kv_write(proj, cols, bias, slots, k_cache, v_cache, heads, kv_heads, dim, vdim):
    if not proj.is_cuda:
        return torch_ref.bias_kv_write(proj, cols, bias, slots, k_cache, v_cache,
                                       heads, kv_heads, dim, vdim)
    return _hip("bias_kv_write").bias_kv_write(
        proj, cols[0], cols[1], cols[2], bias, slots, k_cache, v_cache,
        heads, kv_heads, dim, vdim)


def normed_qkv(proj, p: NormedHeadsParams, positions, slots, k_cache, v_cache):
    """Queries of a fused projection; keys and values go to the cache."""
    if not proj.is_cuda:
        return torch_ref.normed_qkv(proj, p, positions, slots, k_cache, v_cache)
    coef, every = p.temp or (0.0, 1)
    return _hip("normed_qkv").normed_qkv(
        proj, p.q0, p.k0, p.v0, p.q_norm, p.k_norm, p.whole, float(p.eps), p.cos_sin,
        float(coef), every, positions, slots, k_cache, v_cache, p.heads, p.kv_heads,
        p.dim, p.vdim)


def conv_qkv(proj, p: ConvHeadsParams, kv_slots, ring, segments: List[Segment], k_cache,
             v_cache):
    """Convolved and rotated queries [T, heads, DK]; keys and values go to the cache,
    the last projections to the ring."""
    q = torch.empty(proj.shape[0], p.heads, k_cache.shape[3], dtype=proj.dtype,
                    device=proj.device)
    for seg in segments:
        pr, qs, ks = proj[seg.rows], q[seg.rows], kv_slots[seg.rows]
        if not proj.is_cuda:
            torch_ref.conv_qkv(pr, p, ks, ring, seg.cu_or_rows(pr.shape[0]), seg.starts,
                               seg.state_slots, k_cache, v_cache, qs)
            continue
        m = _hip("conv_qkv")
        bseq, boff = (None, None) if seg.decode else seg.block_map(m.conv_qkv_rows())
        m.conv_qkv(pr, p.q0, p.k0, p.v0, p.conv_w, p.turn, p.value_turn, ring, ks, seg.cu,
                   bseq, boff, seg.starts, seg.state_slots, k_cache, v_cache, qs, p.dim,
                   p.vdim)
    return q


def biased_attention(q, k_cache, v_cache, seg: Segment, scale, window, slopes,
                     out, col, vdim, out_scale, log_rate=None, sink=None, chunk: int = 0,
                     turn=None, gate=None):
    """Attention of one segment's rows into out[rows, col:col+heads*vdim]; ``turn``
    and ``gate`` (all rows') act on the result and come without slopes."""
    qs, os_ = q[seg.rows], out[seg.rows]
    gs = None if gate is None else gate[seg.rows]
    if not q.is_cuda:
        torch_ref.biased_attention_paged(
            qs, k_cache, v_cache, seg.block_tables, seg.cu_or_rows(qs.shape[0]),
            seg.context_lens, scale, window, slopes, os_, col, vdim, out_scale,
            log_rate, sink, chunk, turn, gs)
        return
    extra = (scale, window, chunk, slopes, log_rate, sink, turn, gs, os_, col, vdim, out_scale)
    m = _hip("biased_attention")
    matrix = (q.dtype == torch.bfloat16 and q.shape[2] in MATRIX_HEAD_DIMS
              and v_cache.shape[3] in MATRIX_HEAD_DIMS)
    if matrix and seg.decode:
        m.biased_attention_decode(qs, k_cache, v_cache, seg.block_tables,
                                  seg.context_lens, *extra)
    elif matrix:
        rows = m.biased_prefill_rows(q.shape[1] // k_cache.shape[1])
        bseq, boff = seg.block_map(rows, chunk)
        m.biased_attention_prefill(qs, k_cache, v_cache, seg.block_tables, seg.cu,
                                   seg.context_lens, bseq, boff, *extra)
    else:
        bseq, boff = (None, None) if seg.decode else seg.block_map(1)
        m.biased_attention_rows(qs, k_cache, v_cache, seg.block_tables, seg.cu,
                                seg.context_lens, bseq, boff, *extra)


def delta_rule(proj, z, p: DeltaRuleParams, state, conv, seg: Segment,
               out, col, out_scale):
    pr, zs, os_ = proj[seg.rows], z[seg.rows], out[seg.rows]
    if not proj.is_cuda:
        torch_ref.delta_rule(pr, zs, p, state, conv, seg.cu_or_rows(pr.shape[0]),
                             seg.starts, seg.state_slots, os_, col, out_scale)
        return
    m = _hip("delta_rule")
    w = (p.conv_w, p.a_log, p.dt_bias, p.norm)
    sizes = (p.heads, p.kv_heads, p.dim, p.vdim, p.taps, p.q0, p.k0, p.v0, p.b0)
    if seg.decode:
        m.delta_decode(pr, zs, *w, *sizes, p.eps, state, conv, seg.starts,
                       seg.state_slots, os_, col, out_scale)
    else:
        m.delta_prefill(pr, zs, *w, *sizes, p.eps, state, conv, seg.cu,
                        *seg.chunk_map(), seg.starts,
                        seg.state_slots, os_, col, out_scale)


def head_delta_rule(proj, p: HeadDeltaParams, state, conv, seg: Segment, out, col,
                    out_scale):
    pr, os_ = proj[seg.rows], out[seg.rows]
    if not proj.is_cuda:
        torch_ref.head_delta_rule(pr, p, state, conv, seg.cu_or_rows(pr.shape[0]),
                                  seg.starts, seg.state_slots, os_, col, out_scale)
        return
    m = _hip("head_delta_rule")
    args = (pr, p.conv_w, p.a_log, p.dt_bias, p.norm, p.heads, p.kv_heads, p.dim, p.vdim,
            p.taps, p.q0, p.k0, p.v0, p.b0, p.a0, p.g0, p.eps, state, conv)
    if seg.decode:
        m.head_delta_decode(*args, seg.starts, seg.state_slots, os_, col, out_scale)
    else:
        m.head_delta_prefill(*args, seg.cu, *seg.chunk_map(), seg.starts, seg.state_slots,
                             os_, col, out_scale)


def matrix_memory(proj, p: MatrixMemoryParams, state, norm, top, seg: Segment, out, col,
                  out_scale):
    """``state``, ``norm`` and ``top`` hold every slot's memory, normaliser and
    running maximum."""
    pr, os_ = proj[seg.rows], out[seg.rows]
    if not proj.is_cuda:
        torch_ref.matrix_memory(pr, p, state, norm, top, seg.cu_or_rows(pr.shape[0]),
                                seg.starts, seg.state_slots, os_, col, out_scale)
        return
    m = _hip("matrix_memory")
    args = (pr, p.i_bias, p.f_bias, p.norm, p.heads, p.dim, p.vdim, p.q0, p.k0, p.v0,
            p.i0, p.f0, p.g0, p.cap, p.eps, state, norm, top)
    if seg.decode:
        m.memory_decode(*args, seg.starts, seg.state_slots, os_, col, out_scale)
    else:
        m.memory_prefill(*args, seg.cu, *seg.chunk_map(), seg.starts, seg.state_slots,
                         os_, col, out_scale)


def retention(proj, p: RetentionParams, state, seg: Segment, out):
    pr, os_ = proj[seg.rows], out[seg.rows]
    if not proj.is_cuda:
        torch_ref.retention(pr, p, state, seg.cu_or_rows(pr.shape[0]), seg.starts,
                            seg.state_slots, os_)
        return
    m = _hip("retention")
    sizes = (p.heads, p.dim, p.vdim, p.rot_dims, p.q0, p.k0, p.v0, p.g0)
    if seg.decode:
        m.retention_decode(pr, p.decay, p.cos_sin, *sizes, p.eps, state, seg.starts,
                           seg.state_slots, os_)
    else:
        m.retention_prefill(pr, p.decay, p.cos_sin, *sizes, p.eps, state, seg.cu,
                            *seg.chunk_map(), seg.starts, seg.state_slots, os_)


def moe_clamped_glu(h, router, bias, top: int, w_gate_up, w_down, limit: float,
                    alpha: float = 1.702):
    """Routed experts, not yet summed: (y, place, weights) for
    ``residual_rmsnorm``, which adds the weighted rows to the residual."""
    if not h.is_cuda:
        sel, weights = torch_ref.moe_route(h, router, bias, top)
    else:
        sel, weights = _hip("moe_route").moe_route(h, router, bias, top)
    y, place = expert_rows(h, sel, w_gate_up, w_down, limit, alpha, 1.0)
    return y, place, weights


def moe_grouped_glu(h, router, correction, top: int, groups: int, keep: int, scale: float,
                    w_gate_up, w_down):
    """Plain GLU experts chosen by corrected sigmoid scores among the best groups;
    (y, place, weights) for ``output_norm``."""
    if not h.is_cuda:
        sel, weights = torch_ref.moe_route_grouped(h, router, correction, top, groups, keep,
                                                   float(scale))
    else:
        sel, weights = _hip("moe_route_grouped").moe_route_grouped(
            h, router, correction, top, groups, keep, float(scale))
    y, place = expert_rows(h, sel, w_gate_up, w_down, float("inf"), 1.0, 0.0)
    return y, place, weights


def moe_softmax_relu2(h, router, top: int, groups: int, keep: int, scale: float, w_up,
                      w_down):
    """Squared-relu experts chosen and weighed by a softmax over all of them, among
    the groups of the best; (y, place, weights) for the next norm."""
    if not h.is_cuda:
        sel, weights = torch_ref.moe_route_softmax(h, router, top, groups, keep, scale)
        return *torch_ref.moe_relu2(h, sel, w_up, w_down), weights
    m = _hip("moe_relu2")
    sel, weights = m.moe_route_grouped(h, router, None, top, groups, keep, float(scale))
    return *m.moe_relu2(h, sel, w_up, w_down), weights


def expert_rows(h, sel, w_gate_up, w_down, limit: float, alpha: float, shift: float):
    f = torch_ref.moe_clamped_glu if not h.is_cuda else \
        _hip("moe_clamped_glu").moe_clamped_glu
    return f(h, sel, w_gate_up, w_down, float(limit), float(alpha), float(shift))


def output_norm(src, x, weight, bias, eps, delta=None, gate=None, moe=None, depth=None,
                final=None, dtype=None):
    """x = src + layer norm of a sub-layer's result (see ``torch_ref``), with the
    depth average and the final norm that may follow it in the same kernel."""
    if not src.is_cuda:
        return torch_ref.output_norm(src, x, weight, bias, eps, delta, gate, moe, depth,
                                     final, dtype)
    y, place, share = moe if moe is not None else (None, None, None)
    kept, coefs = depth if depth is not None else (None, None)
    fw, fb = final if final is not None else (None, None)
    return _hip("output_norm").output_norm(
        src, x, weight, bias, delta, gate, y, place, share, kept, coefs, fw, fb, float(eps),
        dtype == torch.bfloat16)


def gelu(z):
    """Rows of ``z`` may be strided."""
    return torch_ref.gelu(z) if not z.is_cuda else _hip("gelu").gelu(z)


def relu2(z):
    return torch_ref.relu2(z) if not z.is_cuda else _hip("relu2").relu2(z)


def silu_glu(z, ff: int):
    return torch_ref.silu_glu(z, ff) if not z.is_cuda else _hip("silu_glu").silu_glu(z, ff)
