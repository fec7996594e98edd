"""Token mixers and feed-forwards of the layer-listed decoders.

Every mixer reads the normed hidden state through ONE fused input projection
(all of its projections stacked along the rows, each segment starting at a
multiple of 8 columns so the kernels can load vectors) and ends in one output
projection. The kernels between the two take columns of the fused result.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence, Tuple

import torch
import torch.nn as nn

from .. import ops
from .config import (
    ConvAttentionSpec,
    DenseSpec,
    FusedMixerSpec,
    GroupedMoESpec,
    HeadDeltaSpec,
    LatentAttentionSpec,
    MatrixMemorySpec,
    MoESpec,
    NormedAttentionSpec,
    ParallelMixerSpec,
    RetentionSpec,
    RotationSpec,
)


def _param(*shape, dtype) -> nn.Parameter:
    return nn.Parameter(torch.zeros(*shape, dtype=dtype), requires_grad=False)


def _rotation(rotations: dict, rot: RotationSpec, max_position: int) -> torch.Tensor:
    """The cosines and sines of ``rot``, one table for all layers that share it."""
    if rot not in rotations:
        rotations[rot] = ops.torch_ref.rotation_table(rot.dims, max_position, rot.base,
                                                      rot.yarn)
    return rotations[rot]


class FusedColumns:
    """Row segments of a fused projection weight, by name."""

    ALIGN, TOTAL = 8, 64

    def __init__(self, widths: Sequence[Tuple[str, int]]):
        self.at: Dict[str, int] = {}
        self.width: Dict[str, int] = {}
        n = 0
        for name, w in widths:
            self.at[name], self.width[name] = n, w
            n += -(-w // self.ALIGN) * self.ALIGN
        self.total = -(-n // self.TOTAL) * self.TOTAL

    def pack(self, parts: Dict[str, torch.Tensor], weight: torch.Tensor) -> None:
        """Copy named [rows, in] weights into their segments; padding is zero."""
        weight.zero_()
        for name, t in parts.items():
            assert t.shape == (self.width[name], weight.shape[1]), (name, t.shape)
            weight[self.at[name]:self.at[name] + t.shape[0]].copy_(t)

    def unpack(self, weight: torch.Tensor) -> Dict[str, torch.Tensor]:
        return {n: weight[a:a + self.width[n]] for n, a in self.at.items()}


class ParallelMixer(nn.Module):
    """Distance-biased window attention beside a gated delta rule. Both write
    their heads, already scaled, into one buffer, so the two output
    projections and their sum are a single product."""

    def __init__(self, spec: ParallelMixerSpec, hidden: int, eps: float, dtype):
        super().__init__()
        self.spec = spec
        a, r = spec.left, spec.right
        if a.heads % a.kv_heads or r.heads % r.kv_heads:
            raise ValueError("query heads must be a multiple of key/value heads")
        self.eps = eps
        self.cols = c = FusedColumns([
            ("left.q", a.heads * a.dim), ("left.k", a.kv_heads * a.dim),
            ("left.v", a.kv_heads * a.vdim),
            ("right.q", r.kv_heads * r.dim), ("right.k", r.kv_heads * r.dim),
            ("right.v", r.heads * r.vdim), ("right.b", r.heads),
            ("right.a1", r.decay_rank), ("right.g1", r.gate_rank)])
        # the two low-rank second stages are one block-diagonal product over
        # the adjacent a1 | g1 columns
        self.low = (c.at["right.a1"], c.at["right.g1"] + r.gate_rank)
        self.low_split = c.at["right.g1"] - c.at["right.a1"]
        self.in_proj = _param(c.total, hidden, dtype=dtype)
        self.in_bias = _param(a.heads * a.dim + a.kv_heads * (a.dim + a.vdim),
                              dtype=torch.float32)
        self.low_proj = _param(r.heads * (r.dim + r.vdim), self.low[1] - self.low[0],
                               dtype=dtype)
        self.out_proj = _param(hidden, a.heads * a.vdim + r.heads * r.vdim, dtype=dtype)
        f32 = torch.float32
        self.conv = _param(2 * r.kv_heads * r.dim + r.heads * r.vdim, r.conv, dtype=f32)
        self.a_log = _param(r.heads, dtype=f32)
        self.dt_bias = _param(r.heads * r.dim, dtype=f32)
        self.head_norm = _param(r.vdim, dtype=f32)
        self.register_buffer("slopes", torch.tensor(
            [2.0 ** (-8.0 * (h + 1) / a.heads) for h in range(a.heads)],
            dtype=f32), persistent=False)
        self._delta: Optional[ops.DeltaRuleParams] = None

    def kv_layout(self, dtype, device) -> List[Tuple[int, int, int]]:
        a = self.spec.left
        return [(a.kv_heads, *ops.cache_head_dims(a.dim, a.vdim, dtype, device))]

    def state_layout(self, dtype) -> List[tuple]:
        r = self.spec.right
        return [(((r.heads, r.dim, r.vdim), torch.float32),
                 ((r.conv, self.conv.shape[0]), dtype))]

    def load(self, get) -> None:
        a, r = self.spec.left, self.spec.right
        self.cols.pack({n: get(n) for n in self.cols.at}, self.in_proj)
        self.in_bias.copy_(torch.cat([get(f"left.{n}.b") for n in "qkv"]))
        self.low_proj.zero_()
        nd = r.heads * r.dim
        self.low_proj[:nd, :r.decay_rank].copy_(get("right.a2"))
        self.low_proj[nd:, self.low_split:].copy_(get("right.g2"))
        self.conv.copy_(torch.cat([get(f"right.{n}.conv") for n in "qkv"]))
        self.a_log.copy_(get("right.A_log"))
        self.dt_bias.copy_(get("right.dt_bias"))
        self.head_norm.copy_(get("right.norm"))
        self.out_proj.copy_(torch.cat([get("left.o"), get("right.o")], dim=1))

    def tensors(self) -> Dict[str, torch.Tensor]:
        """Inverse of ``load``: the checkpoint's tensors by name."""
        a, r = self.spec.left, self.spec.right
        out = dict(self.cols.unpack(self.in_proj))
        nq, nk = a.heads * a.dim, a.kv_heads * a.dim
        for n, b in zip("qkv", self.in_bias.split([nq, nk, a.kv_heads * a.vdim])):
            out[f"left.{n}.b"] = b
        nd, ck = r.heads * r.dim, r.kv_heads * r.dim
        out["right.a2"] = self.low_proj[:nd, :r.decay_rank]
        out["right.g2"] = self.low_proj[nd:, self.low_split:]
        for n, w in zip("qkv", self.conv.split([ck, ck, r.heads * r.vdim])):
            out[f"right.{n}.conv"] = w
        out["right.A_log"], out["right.dt_bias"] = self.a_log, self.dt_bias
        out["right.norm"] = self.head_norm
        out["left.o"] = self.out_proj[:, :a.heads * a.vdim]
        out["right.o"] = self.out_proj[:, a.heads * a.vdim:]
        return out

    def init_random(self, randn) -> None:
        hidden = self.in_proj.shape[1]
        r = self.spec.right
        self.load(lambda n: {
            "right.A_log": lambda s: randn(s) * 0.5,
            "right.dt_bias": lambda s: randn(s) - 3.0,
            "right.norm": lambda s: torch.ones(s),
        }.get(n, lambda s: randn(s) * (s[-1] ** -0.5 if len(s) > 1 else 0.1))(
            self._shape(n, hidden)))

    def _shape(self, name: str, hidden: int) -> Tuple[int, ...]:
        a, r = self.spec.left, self.spec.right
        fixed = {
            "left.q.b": (a.heads * a.dim,), "left.k.b": (a.kv_heads * a.dim,),
            "left.v.b": (a.kv_heads * a.vdim,),
            "right.q.conv": (r.kv_heads * r.dim, r.conv),
            "right.k.conv": (r.kv_heads * r.dim, r.conv),
            "right.v.conv": (r.heads * r.vdim, r.conv),
            "right.A_log": (r.heads,), "right.norm": (r.vdim,),
            "right.dt_bias": (r.heads * r.dim,),
            "right.a2": (r.heads * r.dim, r.decay_rank),
            "right.g2": (r.heads * r.vdim, r.gate_rank),
            "left.o": (hidden, a.heads * a.vdim),
            "right.o": (hidden, r.heads * r.vdim)}
        return fixed.get(name) or (self.cols.width[name], hidden)

    def _delta_params(self) -> ops.DeltaRuleParams:
        # built lazily: the tensors move with .to(device)
        if self._delta is None or self._delta.conv_w.device != self.conv.device:
            r, at = self.spec.right, self.cols.at
            self._delta = ops.DeltaRuleParams(
                r.heads, r.kv_heads, r.dim, r.vdim, r.conv, at["right.q"],
                at["right.k"], at["right.v"], at["right.b"], self.conv.data,
                self.a_log.data, self.dt_bias.data, self.head_norm.data, self.eps)
        return self._delta

    def forward(self, h, meta, segments, kv, state):
        a, at = self.spec.left, self.cols.at
        (k_cache, v_cache), (S, conv) = kv[0], state[0]
        proj = ops.linear(h, self.in_proj)
        z = ops.linear(proj[:, self.low[0]:self.low[1]], self.low_proj)
        q = ops.bias_kv_write(
            proj, (at["left.q"], at["left.k"], at["left.v"]), self.in_bias,
            meta.slot_mapping, k_cache, v_cache, a.heads, a.kv_heads, a.dim, a.vdim)
        out = torch.empty(h.shape[0], self.out_proj.shape[1], dtype=h.dtype,
                          device=h.device)
        for seg in segments:
            ops.biased_attention(q, k_cache, v_cache, seg, a.scale, a.window,
                                 self.slopes, out, 0, a.vdim, self.spec.left_scale)
            ops.delta_rule(proj, z, self._delta_params(), S, conv, seg, out,
                           a.heads * a.vdim, self.spec.right_scale)
        return ops.linear(out, self.out_proj)


class RetentionMixer(nn.Module):
    """Fixed-decay linear attention with rotary positions and an output gate."""

    def __init__(self, spec: RetentionSpec, hidden: int, eps: float, dtype,
                 cos_sin: torch.Tensor):
        super().__init__()
        if len(spec.decay) != spec.heads:
            raise ValueError("one decay per head is needed")
        if spec.rot_dims % 2 or spec.rot_dims > spec.dim:
            raise ValueError(f"cannot rotate {spec.rot_dims} of {spec.dim} dimensions")
        self.spec = spec
        self.eps = eps
        n, e = spec.heads * spec.dim, spec.heads * spec.vdim
        self.cols = FusedColumns([("q", n), ("k", n), ("v", e), ("g", e)])
        self.in_proj = _param(self.cols.total, hidden, dtype=dtype)
        self.out_proj = _param(hidden, e, dtype=dtype)
        self.register_buffer("decay", torch.tensor(spec.decay, dtype=torch.float32),
                             persistent=False)
        self.register_buffer("cos_sin", cos_sin, persistent=False)
        self._p: Optional[ops.RetentionParams] = None

    def kv_layout(self, dtype, device) -> List[Tuple[int, int, int]]:
        return []

    def state_layout(self, dtype) -> List[tuple]:
        s = self.spec
        return [(((s.heads, s.dim, s.vdim), torch.float32),)]

    def load(self, get) -> None:
        self.cols.pack({n: get(n) for n in self.cols.at}, self.in_proj)
        self.out_proj.copy_(get("o"))

    def tensors(self) -> Dict[str, torch.Tensor]:
        return {**self.cols.unpack(self.in_proj), "o": self.out_proj}

    def init_random(self, randn) -> None:
        hidden = self.in_proj.shape[1]

        def get(n):
            s = (hidden, self.out_proj.shape[1]) if n == "o" else (self.cols.width[n], hidden)
            return randn(s) * s[-1] ** -0.5

        self.load(get)

    def forward(self, h, meta, segments, kv, state):
        s, at = self.spec, self.cols.at
        if self._p is None or self._p.decay.device != self.decay.device:
            self._p = ops.RetentionParams(
                s.heads, s.dim, s.vdim, s.rot_dims, at["q"], at["k"], at["v"],
                at["g"], self.decay, self.cos_sin, self.eps)
        proj = ops.linear(h, self.in_proj)
        out = torch.empty(h.shape[0], self.out_proj.shape[1], dtype=h.dtype,
                          device=h.device)
        for seg in segments:
            ops.retention(proj, self._p, state[0][0], seg, out)
        return ops.linear(out, self.out_proj)


class LatentAttention(nn.Module):
    """Attention over one cached latent per token: keys and values are per-head
    linear maps of it, and a part of every key that the heads share may be rotated
    by its position and cached beside it. Queries come straight from the input or
    through a normed latent of their own; the softmax may have a sink, every head a
    sigmoid gate, and there may be a window. A layer may read an earlier layer's
    latents instead of its own. Heads and latents are padded with zeros to the
    kernels' widths."""

    def __init__(self, spec: LatentAttentionSpec, hidden: int, eps: float, dtype,
                 max_position: int, rotations: dict):
        super().__init__()
        self.spec = spec
        self.eps = eps
        H, R = spec.heads, ops.latent_width(spec.kv_rank)
        rot = spec.rot.dims if spec.rot else 0
        if rot:
            D, self.tail, key = ops.latent_rotary_widths(spec.dim, rot)
            cos_sin = _rotation(rotations, spec.rot, max_position)
        else:
            D, self.tail, key, cos_sin = ops.latent_head_width(spec.dim), 0, 0, None
        E = ops.latent_head_width(spec.vdim)
        self.D, self.E, self.R, self.row = D, E, R, R + key
        self.own = spec.kv_from is None
        columns = [("dq", spec.q_rank)] if spec.q_rank else [("q", H * (D + self.tail))]
        if self.own:
            columns += [("dkv", spec.kv_rank)] + ([("kr", rot)] if rot else [])
        if spec.gate:
            columns.append(("g", H))
        self.cols = FusedColumns(columns)
        f32 = torch.float32
        self.in_proj = _param(self.cols.total, hidden, dtype=dtype)
        if spec.q_rank:
            self.q_norm = _param(spec.q_rank, dtype=f32)
            self.uq = _param(H * (D + self.tail), spec.q_rank, dtype=dtype)
        if self.own:
            self.latent_norm = _param(spec.kv_rank, dtype=f32)
        self.uk = _param(H, D, R, dtype=dtype)
        self.uk_t = _param(H, R, D, dtype=dtype)
        self.uv = _param(H, E, R, dtype=dtype)
        self.sink = _param(H, dtype=f32) if spec.sink else None
        self.out_proj = _param(hidden, H * E, dtype=dtype)
        self.register_buffer("cos_sin", cos_sin, persistent=False)
        self._p: Optional[ops.LatentParams] = None

    def kv_layout(self, dtype, device) -> List[Tuple[int, int, int]]:
        return [(1, self.row, 0)] if self.own else []

    def state_layout(self, dtype) -> List[tuple]:
        return []

    def _query_rows(self) -> torch.Tensor:
        """The queries' weights [H, D + tail, in]."""
        w = self.uq if self.spec.q_rank else self.cols.unpack(self.in_proj)["q"]
        return w.unflatten(0, (self.spec.heads, self.D + self.tail))

    def load(self, get) -> None:
        s, H, dev = self.spec, self.spec.heads, self.uk.device
        rot = s.rot.dims if s.rot else 0

        def heads(t, n):  # [H*n, ...] -> [H, n, ...]
            return t.to(dev).unflatten(0, (H, n))

        self.in_proj.zero_()
        parts = self.cols.unpack(self.in_proj)
        queries, q = self._query_rows(), heads(get("uq" if s.q_rank else "q"), s.dim + rot)
        queries.zero_()
        queries[:, :s.dim] = q[:, :s.dim].to(queries.dtype)
        queries[:, self.D:self.D + rot] = q[:, s.dim:].to(queries.dtype)
        if s.q_rank:
            parts["dq"].copy_(get("dq"))
            self.q_norm.copy_(get("dq.norm"))
        if self.own:
            dkv = get("dkv")
            parts["dkv"].copy_(dkv[:s.kv_rank])
            if rot:
                parts["kr"].copy_(dkv[s.kv_rank:])
            self.latent_norm.copy_(get("dkv.norm"))
        if s.gate:
            parts["g"].copy_(get("g"))
        self.uk.zero_()
        self.uv.zero_()
        self.uk[:, :s.dim, :s.kv_rank] = heads(get("uk"), s.dim).to(self.uk.dtype)
        self.uv[:, :s.vdim, :s.kv_rank] = heads(get("uv"), s.vdim).to(self.uv.dtype)
        self.uk_t.copy_(self.uk.transpose(1, 2))
        if s.sink:
            self.sink.copy_(get("sink"))
        self.out_proj.zero_()
        self.out_proj.unflatten(1, (H, self.E))[:, :, :s.vdim] = get("o").to(
            device=dev, dtype=self.out_proj.dtype).unflatten(1, (H, s.vdim))

    def tensors(self) -> Dict[str, torch.Tensor]:
        s, H = self.spec, self.spec.heads
        rot = s.rot.dims if s.rot else 0
        parts, q = self.cols.unpack(self.in_proj), self._query_rows()
        q = torch.cat([q[:, :s.dim], q[:, self.D:self.D + rot]], 1).flatten(0, 1)
        out = {"uq": q, "dq": parts["dq"], "dq.norm": self.q_norm} if s.q_rank else {"q": q}
        if self.own:
            out["dkv"] = torch.cat([parts[n] for n in ("dkv", "kr") if n in parts])
            out["dkv.norm"] = self.latent_norm
        if s.gate:
            out["g"] = parts["g"]
        out["uk"] = self.uk[:, :s.dim, :s.kv_rank].flatten(0, 1)
        out["uv"] = self.uv[:, :s.vdim, :s.kv_rank].flatten(0, 1)
        if s.sink:
            out["sink"] = self.sink
        out["o"] = self.out_proj.unflatten(1, (H, self.E))[:, :, :s.vdim].flatten(1)
        return out

    def init_random(self, randn) -> None:
        shapes = {n: tuple(t.shape) for n, t in self.tensors().items()}
        self.load(lambda n: randn(shapes[n]) * shapes[n][1] ** -0.5 if len(shapes[n]) > 1
                  else 1.0 + 0.1 * randn(shapes[n]) if n.endswith(".norm")
                  else randn(shapes[n]))

    def _params(self):
        # built lazily: the tensors move with .to(device)
        if self._p is None or self._p[0].uk.device != self.uk.device:
            s, at = self.spec, self.cols.at
            front = None
            if s.q_rank or self.own:
                front = ops.LatentFrontParams(
                    at.get("dkv"), s.kv_rank, self.latent_norm.data if self.own else None,
                    self.eps, at.get("kr", 0), self.R, self.cos_sin, at.get("dq", 0),
                    s.q_rank, self.q_norm.data if s.q_rank else None)
            self._p = (ops.LatentParams(
                s.heads, self.D, self.E, s.scale, at.get("q", 0), at.get("g"), self.uk.data,
                self.uk_t.data, self.uv.data, self.sink.data if s.sink else None, self.tail,
                self.cos_sin, s.window), front)
        return self._p

    def forward(self, h, meta, segments, kv, state):
        p, front = self._params()
        cache, H, width = kv[0][0], self.spec.heads, self.D + self.tail
        proj, q = ops.linear(h, self.in_proj), None
        if front is not None:
            q = ops.latent_front(proj, front, meta.positions, meta.slot_mapping, cache)
        if q is not None:
            q = ops.linear(q, self.uq).unflatten(1, (H, width))
        elif self.tail:
            q = proj[:, p.q0:p.q0 + H * width].unflatten(1, (H, width))
        out = torch.empty(h.shape[0], self.out_proj.shape[1], dtype=h.dtype,
                          device=h.device)
        for seg in segments:
            ops.latent_attention(proj, p, cache, seg, out, q, meta.positions)
        return ops.linear(out, self.out_proj)


class MixerPart(nn.Module):
    """One of the mixers a ``FusedMixer`` runs side by side: its columns of the
    common input projection, weights of its own, and heads for the common output
    projection."""

    #: names of the checkpoint's tensors beside projections and "o", with their
    #: shapes; each is held as the fp32 parameter of the same place in ``own``
    shapes: Dict[str, Tuple[int, ...]]

    def __init__(self, spec, columns: Sequence[Tuple[str, int]], out_width: int,
                 shapes: Dict[str, Tuple[int, ...]]):
        super().__init__()
        self.spec = spec
        self.columns = list(columns)
        self.out_width = out_width
        self.shapes = shapes
        self.own = nn.ParameterList([_param(*s, dtype=torch.float32)
                                     for s in shapes.values()])
        self._p = None

    def kv_layout(self, dtype, device) -> List[Tuple[int, int, int]]:
        return []

    def state_layout(self, dtype) -> List[tuple]:
        return []

    def tensors(self) -> Dict[str, torch.Tensor]:
        return dict(zip(self.shapes, self.own))

    def random(self, name: str, randn) -> torch.Tensor:
        """A random tensor of ``shapes``."""
        return 1.0 + 0.1 * randn(self.shapes[name])

    def params(self, at: Dict[str, int], eps: float):
        """The kernels' sizes, columns and weights; built lazily, for the tensors
        move with .to(device)."""
        if self._p is None or self._device != self.own[0].device:
            self._device = self.own[0].device
            self._p = self.make_params(
                at, {n: t.data for n, t in self.tensors().items()}, eps)
        return self._p


class NormedAttention(MixerPart):
    """Grouped-query attention over normed queries and keys, with rotary
    positions or a logarithmic distance bias, query temperature and sink."""

    def __init__(self, spec: NormedAttentionSpec, max_position: int, rotations: dict):
        H, G, d, e = spec.heads, spec.kv_heads, spec.dim, spec.vdim
        columns = [("q", H * d), ("k", G * d)]
        if not spec.shared_kv:
            columns.append(("v", G * e))
        if spec.norm not in ("head", "whole"):
            raise ValueError(f"unknown norm of queries and keys {spec.norm!r}")
        whole = spec.norm == "whole"
        shapes = {"q.norm": (H * d if whole else d,), "k.norm": (G * d if whole else d,)}
        if spec.log_bias:
            shapes["r1"] = shapes["r2"] = (H,)
        super().__init__(spec, columns, H * e, shapes)
        cos_sin = None
        if spec.rot_dims:
            key = (spec.rot_dims, spec.rot_base)
            if key not in rotations:  # one table for all layers that share it
                rotations[key] = ops.torch_ref.rope_cos_sin_cache(
                    spec.rot_dims, max_position, spec.rot_base)
            cos_sin = rotations[key]
        self.register_buffer("cos_sin", cos_sin, persistent=False)
        zeros = torch.zeros(H, dtype=torch.float32)
        self.register_buffer("flat", None if spec.log_bias else zeros, persistent=False)
        self.register_buffer("sink", zeros.clone() if spec.sink else None, persistent=False)

    def kv_layout(self, dtype, device):
        s = self.spec
        return [(s.kv_heads, *ops.cache_head_dims(s.dim, s.vdim, dtype, device))]

    def random(self, name, randn):
        # distances that matter, of every reach
        return randn(self.shapes[name]).abs() if name in ("r1", "r2") \
            else super().random(name, randn)

    def make_params(self, at, t, eps):
        s = self.spec
        heads = ops.NormedHeadsParams(
            s.heads, s.kv_heads, s.dim, s.vdim, at["q"], at["k"],
            at["k" if s.shared_kv else "v"], t["q.norm"], t["k.norm"], s.norm == "whole",
            eps, self.cos_sin, s.q_temp)
        return heads, t.get("r1", self.flat), t.get("r2")

    def forward(self, proj, at, eps, meta, segments, kv, state, out, col, scale):
        s = self.spec
        heads, slopes, rate = self.params(at, eps)
        k_cache, v_cache = kv[0]
        q = ops.normed_qkv(proj, heads, meta.positions, meta.slot_mapping, k_cache, v_cache)
        for seg in segments:
            ops.biased_attention(q, k_cache, v_cache, seg, s.scale, 0, slopes, out, col,
                                 s.vdim, scale, rate, self.sink)


class ConvAttention(MixerPart):
    """Grouped-query attention over convolved projections with rotary positions on
    queries and keys, and on values too if they turn; in windows or chunks, with a
    sink, and a sigmoid gate of every output channel."""

    def __init__(self, spec: ConvAttentionSpec, max_position: int, rotations: dict):
        H, G, d, e = spec.heads, spec.kv_heads, spec.dim, spec.vdim
        columns = [("q", H * d), ("k", G * d), ("v", G * e)]
        shapes = {f"{n}.conv": (w, spec.conv) for n, w in columns}
        if spec.gate:
            columns.append(("g", H * e))
        super().__init__(spec, columns, H * e, shapes)
        self.register_buffer("turn", _rotation(rotations, spec.rot, max_position),
                             persistent=False)
        self.register_buffer("value_turn", _rotation(
            rotations, RotationSpec(e, spec.value_base), max_position)
            if spec.value_base else None, persistent=False)
        self.register_buffer("sink", torch.zeros(H, dtype=torch.float32)
                             if spec.sink else None, persistent=False)

    def kv_layout(self, dtype, device):
        s = self.spec
        return [(s.kv_heads, *ops.cache_head_dims(s.dim, s.vdim, dtype, device))]

    def state_layout(self, dtype):
        s = self.spec
        channels = s.heads * s.dim + s.kv_heads * (s.dim + s.vdim)
        return [(((s.conv - 1, channels), dtype),)]

    def random(self, name, randn):
        return randn(self.shapes[name]) * self.spec.conv ** -0.5

    def make_params(self, at, t, eps):
        s = self.spec
        return ops.ConvHeadsParams(
            s.heads, s.kv_heads, s.dim, s.vdim, at["q"], at["k"], at["v"],
            torch.cat([t[f"{n}.conv"] for n in "qkv"]).t().contiguous(), self.turn,
            self.value_turn)

    def forward(self, proj, at, eps, meta, segments, kv, state, out, col, scale):
        s, (k_cache, v_cache) = self.spec, kv[0]
        q = ops.conv_qkv(proj, self.params(at, eps), meta.slot_mapping, state[0][0], segments,
                         k_cache, v_cache)
        gate = proj[:, at["g"]:at["g"] + s.heads * s.vdim] if s.gate else None
        for seg in segments:
            ops.biased_attention(q, k_cache, v_cache, seg, s.scale, s.window, None, out, col,
                                 s.vdim, scale, sink=self.sink, chunk=s.chunk,
                                 turn=self.value_turn, gate=gate)


class HeadDelta(MixerPart):
    """Gated delta rule with one decay per head."""

    def __init__(self, spec: HeadDeltaSpec):
        H, ck, cv = spec.heads, spec.kv_heads * spec.dim, spec.heads * spec.vdim
        super().__init__(
            spec, [("q", ck), ("k", ck), ("v", cv), ("b", H), ("a", H), ("g", cv)], cv,
            {"q.conv": (ck, spec.conv), "k.conv": (ck, spec.conv), "v.conv": (cv, spec.conv),
             "A_log": (H,), "dt_bias": (H,), "norm": (spec.vdim,)})

    def state_layout(self, dtype):
        s = self.spec
        channels = 2 * s.kv_heads * s.dim + s.heads * s.vdim
        return [(((s.heads, s.dim, s.vdim), torch.float32), ((s.conv, channels), dtype))]

    def random(self, name, randn):
        x = randn(self.shapes[name])
        return {"A_log": x * 0.5, "dt_bias": x - 3.0, "norm": 1.0 + 0.1 * x}.get(
            name, x * self.spec.conv ** -0.5)

    def make_params(self, at, t, eps):
        s = self.spec
        return ops.HeadDeltaParams(
            s.heads, s.kv_heads, s.dim, s.vdim, s.conv, *(at[n] for n in "qkvbag"),
            torch.cat([t[f"{n}.conv"] for n in "qkv"]), t["A_log"], t["dt_bias"], t["norm"],
            eps)

    def forward(self, proj, at, eps, meta, segments, kv, state, out, col, scale):
        p = self.params(at, eps)
        for seg in segments:
            ops.head_delta_rule(proj, p, *state[0], seg, out, col, scale)


class MatrixMemory(MixerPart):
    """mLSTM: a decaying sum of key-value products with exponential input gates,
    read through its normaliser."""

    def __init__(self, spec: MatrixMemorySpec):
        H, n, e = spec.heads, spec.heads * spec.dim, spec.heads * spec.vdim
        super().__init__(
            spec, [("q", n), ("k", n), ("v", e), ("i", H), ("f", H), ("g", e)], e,
            {"i.b": (H,), "f.b": (H,), "norm": (e,)})

    def state_layout(self, dtype):
        s, f32 = self.spec, torch.float32
        return [(((s.heads, s.dim, s.vdim), f32), ((s.heads, s.dim), f32), ((s.heads,), f32))]

    def random(self, name, randn):
        x = randn(self.shapes[name])
        return {"i.b": x, "f.b": x + 4.0}.get(name, 1.0 + 0.1 * x)

    def make_params(self, at, t, eps):
        s = self.spec
        return ops.MatrixMemoryParams(
            s.heads, s.dim, s.vdim, *(at[n] for n in "qkvifg"), t["i.b"], t["f.b"],
            t["norm"], s.gate_cap, eps)

    def forward(self, proj, at, eps, meta, segments, kv, state, out, col, scale):
        p = self.params(at, eps)
        for seg in segments:
            ops.matrix_memory(proj, p, *state[0], seg, out, col, scale)


class FusedMixer(nn.Module):
    """Parts side by side. All read one fused input projection and write their
    scaled heads into one buffer, so the output projections and their sum are a
    single product."""

    def __init__(self, spec: FusedMixerSpec, hidden: int, eps: float, dtype,
                 max_position: int, rotations: dict):
        super().__init__()
        self.eps = eps
        self.names = [name for name, _, _ in spec.parts]
        self.scales = [scale for _, _, scale in spec.parts]
        make = {NormedAttentionSpec: lambda s: NormedAttention(s, max_position, rotations),
                ConvAttentionSpec: lambda s: ConvAttention(s, max_position, rotations),
                HeadDeltaSpec: HeadDelta, MatrixMemorySpec: MatrixMemory}
        self.parts = nn.ModuleList([make[type(s)](s) for _, s, _ in spec.parts])
        self.cols = FusedColumns([(name + n, w) for name, part in zip(self.names, self.parts)
                                  for n, w in part.columns])
        #: each part's columns under its own names
        self.at = [{n: self.cols.at[name + n] for n, _ in part.columns}
                   for name, part in zip(self.names, self.parts)]
        self.in_proj = _param(self.cols.total, hidden, dtype=dtype)
        self.out_proj = _param(hidden, sum(p.out_width for p in self.parts), dtype=dtype)

    def kv_layout(self, dtype, device) -> List[Tuple[int, int, int]]:
        return [e for p in self.parts for e in p.kv_layout(dtype, device)]

    def state_layout(self, dtype) -> List[tuple]:
        return [e for p in self.parts for e in p.state_layout(dtype)]

    def load(self, get) -> None:
        self.cols.pack({n: get(n) for n in self.cols.at}, self.in_proj)
        for name, part in zip(self.names, self.parts):
            for n, t in part.tensors().items():
                t.copy_(get(name + n))
        self.out_proj.copy_(torch.cat([get(name + "o") for name in self.names], dim=1))

    def tensors(self) -> Dict[str, torch.Tensor]:
        out = dict(self.cols.unpack(self.in_proj))
        for name, part, o in zip(self.names, self.parts, self.out_proj.split(
                [p.out_width for p in self.parts], dim=1)):
            out.update({name + n: t for n, t in part.tensors().items()})
            out[name + "o"] = o
        return out

    def init_random(self, randn) -> None:
        hidden = self.out_proj.shape[0]
        made = {}
        for name, part in zip(self.names, self.parts):
            made.update({name + n: part.random(n, randn) for n in part.shapes})
            made[name + "o"] = randn((hidden, part.out_width)) * part.out_width ** -0.5
        self.load(lambda n: made[n] if n in made
                  else randn((self.cols.width[n], hidden)) * hidden ** -0.5)

    def forward(self, h, meta, segments, kv, state):
        proj = ops.linear(h, self.in_proj)
        out = torch.empty(h.shape[0], self.out_proj.shape[1], dtype=h.dtype,
                          device=h.device)
        col = k0 = s0 = 0
        for part, at, scale in zip(self.parts, self.at, self.scales):
            k1 = k0 + len(part.kv_layout(h.dtype, h.device))
            s1 = s0 + len(part.state_layout(h.dtype))
            part(proj, at, self.eps, meta, segments, kv[k0:k1], state[s0:s1], out, col, scale)
            col, k0, s0 = col + part.out_width, k1, s1
        return ops.linear(out, self.out_proj)


class DenseXieluMLP(nn.Module):
    """Two matrices around an xIELU. With ``gated``, the residual gate's
    projection of the same input shares the first product."""

    def __init__(self, spec: DenseSpec, hidden: int, dtype, gated: bool):
        super().__init__()
        self.spec = spec
        self.cols = FusedColumns(([("gate", hidden)] if gated else []) + [("up", spec.ff)])
        self.in_proj = _param(self.cols.total, hidden, dtype=dtype)
        self.gate_bias = _param(hidden, dtype=torch.float32) if gated else None
        self.down = _param(hidden, spec.ff, dtype=dtype)
        self.act = _param(2, dtype=torch.float32)

    def load(self, get, get_gate=None) -> None:
        """``get_gate`` reads the residual gate: its weight, and with ".b" its bias."""
        parts = {"up": get("up")}
        if self.gate_bias is not None:
            parts["gate"] = get_gate("")
            self.gate_bias.copy_(get_gate(".b"))
        self.cols.pack(parts, self.in_proj)
        self.down.copy_(get("down"))
        self.act.copy_(get("act"))

    def tensors(self) -> Dict[str, torch.Tensor]:
        return {"up": self.cols.unpack(self.in_proj)["up"], "down": self.down,
                "act": self.act}

    def gate_tensors(self) -> Dict[str, torch.Tensor]:
        return {"": self.cols.unpack(self.in_proj)["gate"], ".b": self.gate_bias}

    def init_random(self, randn) -> None:
        hidden, ff = self.down.shape
        self.load(lambda n: {"up": lambda: randn((ff, hidden)) * hidden ** -0.5,
                             "down": lambda: randn((hidden, ff)) * ff ** -0.5,
                             "act": lambda: randn((2,)) * 0.5}[n](),
                  lambda n: randn((hidden,)) if n else randn((hidden, hidden)) * hidden ** -0.5)

    def forward(self, h) -> Dict[str, object]:
        at, ff = self.cols.at, self.spec.ff
        z = ops.linear(h, self.in_proj)
        add: Dict[str, object] = {
            "delta": ops.linear(ops.xielu(z[:, at["up"]:at["up"] + ff], self.act), self.down)}
        if self.gate_bias is not None:
            add["gate"] = (z[:, :h.shape[1]], self.gate_bias)
        return add


class DenseGeluMLP(nn.Module):
    """Two matrices around an exact gelu."""

    def __init__(self, spec: DenseSpec, hidden: int, dtype):
        super().__init__()
        self.up = _param(spec.ff, hidden, dtype=dtype)
        self.down = _param(hidden, spec.ff, dtype=dtype)

    def load(self, get) -> None:
        self.up.copy_(get("up"))
        self.down.copy_(get("down"))

    def tensors(self) -> Dict[str, torch.Tensor]:
        return {"up": self.up, "down": self.down}

    def init_random(self, randn) -> None:
        self.load(lambda n: randn(tuple(getattr(self, n).shape))
                  * getattr(self, n).shape[1] ** -0.5)

    def forward(self, h) -> Dict[str, object]:
        return {"delta": ops.linear(ops.gelu(ops.linear(h, self.up)), self.down)}


class RoutedGLU(nn.Module):
    """Top-k routed clamped-GLU experts with a biased fp32 router. Returns the
    chosen experts' rows unsummed; the next residual norm adds them up."""

    ALPHA = 1.702

    def __init__(self, spec: MoESpec, hidden: int, dtype):
        super().__init__()
        self.spec = spec
        self.router = _param(spec.experts, hidden, dtype=dtype)
        self.router_bias = _param(spec.experts, dtype=torch.float32)
        self.gate_up = _param(spec.experts, 2 * spec.ff, hidden, dtype=dtype)
        self.down = _param(spec.experts, hidden, spec.ff, dtype=dtype)

    def load(self, get) -> None:
        self.router.copy_(get("router"))
        self.router_bias.copy_(get("router.b"))
        ff = self.spec.ff
        for e in range(self.spec.experts):
            self.gate_up[e, :ff].copy_(get(f"e{e}.gate"))
            self.gate_up[e, ff:].copy_(get(f"e{e}.up"))
            self.down[e].copy_(get(f"e{e}.down"))

    def tensors(self) -> Dict[str, torch.Tensor]:
        ff = self.spec.ff
        out = {"router": self.router, "router.b": self.router_bias}
        for e in range(self.spec.experts):
            out[f"e{e}.gate"] = self.gate_up[e, :ff]
            out[f"e{e}.up"] = self.gate_up[e, ff:]
            out[f"e{e}.down"] = self.down[e]
        return out

    def init_random(self, randn) -> None:
        hidden, ff = self.router.shape[1], self.spec.ff
        self.router.copy_(randn((self.spec.experts, hidden)) * hidden ** -0.5)
        self.router_bias.copy_(randn((self.spec.experts,)) * 0.1)
        for e in range(self.spec.experts):
            self.gate_up[e].copy_(randn((2 * ff, hidden)) * hidden ** -0.5)
            self.down[e].copy_(randn((hidden, ff)) * ff ** -0.5)

    def forward(self, h) -> Dict[str, object]:
        s = self.spec
        return {"moe": ops.moe_clamped_glu(h, self.router, self.router_bias, s.top,
                                           self.gate_up, self.down, s.limit, self.ALPHA)}


class GroupedExperts(nn.Module):
    """Experts chosen among the best groups, beside a shared expert whose gate, if it
    has one, is one more row of its first product. Returns the chosen rows unsummed;
    the next norm adds everything up."""

    def __init__(self, spec: GroupedMoESpec, hidden: int, dtype):
        super().__init__()
        self.spec = spec
        E, ff, sf = spec.experts, spec.ff, spec.shared_ff
        self.first = ("gate", "up") if spec.act == "silu_glu" else ("up",)
        n = len(self.first)
        self.router = _param(E, hidden, dtype=dtype)
        self.correction = _param(E, dtype=torch.float32) if spec.scores == "sigmoid" else None
        self.up = _param(E, n * ff, hidden, dtype=dtype)
        self.down = _param(E, hidden, ff, dtype=dtype)
        if sf:
            # [gate; up; the shared gate's row; zeros]
            self.shared_in = _param(-(-(n * sf + spec.shared_gate) // 64) * 64, hidden,
                                    dtype=dtype)
            self.shared_down = _param(hidden, sf, dtype=dtype)

    def tensors(self) -> Dict[str, torch.Tensor]:
        """Weights by the checkpoint's names; views that ``load`` fills."""
        s, ff, sf = self.spec, self.spec.ff, self.spec.shared_ff
        out = {"router": self.router}
        if self.correction is not None:
            out["correction"] = self.correction
        for e in range(s.experts):
            for i, name in enumerate(self.first):
                out[f"e{e}.{name}"] = self.up[e, i * ff:(i + 1) * ff]
            out[f"e{e}.down"] = self.down[e]
        if sf:
            for i, name in enumerate(self.first):
                out[f"shared.{name}"] = self.shared_in[i * sf:(i + 1) * sf]
            if s.shared_gate:
                n = len(self.first) * sf
                out["shared.sg"] = self.shared_in[n:n + 1]
            out["shared.down"] = self.shared_down
        return out

    def load(self, get) -> None:
        for name, t in self.tensors().items():
            t.copy_(get(name))

    def init_random(self, randn) -> None:
        tensors = self.tensors()
        self.load(lambda n: randn(tuple(tensors[n].shape))
                  * (0.1 if n == "correction" else tensors[n].shape[1] ** -0.5))

    def forward(self, h) -> Dict[str, object]:
        s = self.spec
        glu, sf = s.act == "silu_glu", s.shared_ff
        if (s.scores == "sigmoid") != glu:
            raise NotImplementedError(f"{s.act} experts behind a {s.scores} router")
        add: Dict[str, object] = {"moe": ops.moe_grouped_glu(
            h, self.router, self.correction, s.top, s.groups, s.keep, s.scale, self.up,
            self.down) if glu else ops.moe_softmax_relu2(
            h, self.router, s.top, s.groups, s.keep, s.scale, self.up, self.down)}
        if sf:
            z = ops.linear(h, self.shared_in)
            a = ops.silu_glu(z, sf) if glu else ops.relu2(z[:, :sf])
            add["delta"] = ops.linear(a, self.shared_down)
            if s.shared_gate:
                add["gate"] = z[:, len(self.first) * sf]
        return add
