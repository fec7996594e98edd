"""Model specs for the families the framework serves.

The reference outsources all model capability to provider APIs
(reference: server/chat/backend/agent/llm.py:32-67 — a registry of rented
models); here the registry is of locally-served architectures.  Weights are
random-initialised in this environment (no network); real deployments load
safetensors checkpoints via models.loader.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Dict, List, Optional, Sequence, Tuple, Union


@dataclass
class ModelSpec:
    name: str
    hidden_size: int
    n_layers: int
    n_heads: int
    n_kv_heads: int
    head_dim: int
    intermediate_size: int
    vocab_size: int
    rope_theta: float = 500000.0
    rms_eps: float = 1e-5
    max_position: int = 131072
    tie_embeddings: bool = False
    # MoE (Mixtral-style); n_experts == 0 => dense MLP
    n_experts: int = 0
    experts_per_token: int = 2
    # Qwen2-family attention projections carry a bias (q/k/v only)
    qkv_bias: bool = False
    # encoder-only (BGE-style) models use bidirectional attention + pooling
    is_encoder: bool = False
    arch: str = "llama"

    @property
    def q_size(self) -> int:
        return self.n_heads * self.head_dim

    @property
    def kv_size(self) -> int:
        return self.n_kv_heads * self.head_dim

    def param_count(self) -> int:
        h, i, v, L = self.hidden_size, self.intermediate_size, self.vocab_size, self.n_layers
        attn = h * (self.q_size + 2 * self.kv_size) + self.q_size * h
        mlp = 3 * h * i if self.n_experts == 0 else self.n_experts * 3 * h * i
        emb = v * h * (1 if self.tie_embeddings else 2)
        return L * (attn + mlp) + emb


# ---- layer-listed decoders -------------------------------------------------
# A HybridSpec spells its layers out one by one: each has a mixer (attention
# beside a recurrence, a recurrence or attention alone) and an optional
# feed-forward. What all layers share (the norms' kind and place, residual gates,
# the convolution of a sublayer's input, depth averages) are fields of the
# HybridSpec.

@dataclass(frozen=True)
class YarnSpec:
    """Frequencies stretched for longer contexts: pairs that turn fewer than
    ``slow`` times within ``original`` positions by ``factor``, pairs that turn more
    than ``fast`` times not at all, those between in part."""
    factor: float
    original: float
    fast: float
    slow: float


@dataclass(frozen=True)
class RotationSpec:
    """Rotary positions of neighbours: dimensions 2i and 2i + 1 of the first ``dims``
    turn by position * base^(-2i/dims)."""
    dims: int
    base: float
    yarn: Optional[YarnSpec] = None

    def __post_init__(self):
        if self.dims < 2 or self.dims % 2:
            raise ValueError(f"cannot rotate {self.dims} dimensions")


@dataclass(frozen=True)
class BiasedAttentionSpec:
    """Grouped-query attention with a per-head linear distance penalty."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int = 0  # keys a query sees, itself included; 0 = all before it


@dataclass(frozen=True)
class DeltaRuleSpec:
    """Gated delta rule with a short convolution and per-channel decay."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: int
    gate_rank: int


@dataclass(frozen=True)
class ParallelMixerSpec:
    left: BiasedAttentionSpec
    right: DeltaRuleSpec
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class RetentionSpec:
    """Linear attention with one fixed decay per head and rotary positions."""
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]
    rot_dims: int
    rot_base: float


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Attention over one cached latent per token."""
    heads: int
    dim: int
    vdim: int
    kv_rank: int
    scale: float
    kv_from: Optional[int] = None  # layer whose latents it reads; None: its own
    q_rank: int = 0     # width of the normed latent queries come from; 0: none
    #: beside the ``dim`` dimensions without positions a head has rot.dims rotated
    #: ones, whose key all heads share; None: no positions
    rot: Optional[RotationSpec] = None
    window: int = 0     # keys a query sees, itself included; 0 = all before it
    sink: bool = True   # a learned term of the softmax's denominator per head
    gate: bool = True   # a sigmoid gate per head


@dataclass(frozen=True)
class NormedAttentionSpec:
    """Grouped-query attention over normed queries and keys."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    norm: str = "head"  # RMS over each "head", or over the "whole" projection
    rot_dims: int = 0   # leading dimensions of a head that rotate; 0: none
    rot_base: float = 1e4
    #: query at position p times 1 + coef ln(floor((p + 1) / every) + 1)
    q_temp: Optional[Tuple[float, int]] = None
    #: values are the keys as projected, before norm and rotation
    shared_kv: bool = False
    #: a_h ln(1 + b_h (i - j)) off the score, with two learned numbers per head
    log_bias: bool = False
    sink: bool = False  # the softmax's denominator has one more term, 1

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError("query heads must be a multiple of key/value heads")
        if self.shared_kv and self.vdim != self.dim:
            raise ValueError("values that are the keys are as wide as the keys")
        if self.rot_dims % 2 or self.rot_dims > self.dim:
            raise ValueError(f"cannot rotate {self.rot_dims} of {self.dim} dimensions")


@dataclass(frozen=True)
class ConvAttentionSpec:
    """Grouped-query attention whose projections pass a short causal convolution."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    conv: int                  # taps
    rot: RotationSpec
    #: values turn with their own position and every head's result back by the
    #: query's, pair m by base^(-2m/vdim) per position; 0: they do not turn
    value_base: float = 0.0
    window: int = 0            # keys a query sees, itself included; 0: no window
    chunk: int = 0             # keys of the query's chunk of positions alone; 0: no chunks
    sink: bool = False         # the softmax's denominator has one more term, 1
    gate: bool = False         # a sigmoid gate as wide as the heads

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError("query heads must be a multiple of key/value heads")
        if self.rot.dims > self.dim:
            raise ValueError(f"cannot rotate {self.rot.dims} of {self.dim} dimensions")
        if self.value_base and self.vdim % 2:
            raise ValueError(f"cannot rotate {self.vdim} value dimensions")
        if self.conv < 1:
            raise ValueError(f"a convolution of {self.conv} taps")


@dataclass(frozen=True)
class HeadDeltaSpec:
    """Gated delta rule with a short convolution, one decay per head and a silu
    gate as wide as the heads."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError("value heads must be a multiple of query/key heads")


@dataclass(frozen=True)
class MatrixMemorySpec:
    """Matrix memory with exponential input and sigmoid forget gates (mLSTM);
    both gates' pre-activations are soft-capped."""
    heads: int
    dim: int
    vdim: int
    gate_cap: float


PartSpec = Union[NormedAttentionSpec, ConvAttentionSpec, HeadDeltaSpec, MatrixMemorySpec]


@dataclass(frozen=True)
class FusedMixerSpec:
    """Parts side by side over one input; their scaled results add up. Each part
    is (prefix of its tensors' names, spec, scale)."""
    parts: Tuple[Tuple[str, PartSpec, float], ...]


@dataclass(frozen=True)
class MoESpec:
    """Softmax-routed clamped GLU experts."""
    experts: int
    top: int
    ff: int
    limit: float


@dataclass(frozen=True)
class GroupedMoESpec:
    """Experts chosen among the best ``keep`` of ``groups`` groups of neighbours,
    beside a shared expert (of width ``shared_ff``; 0: none)."""
    experts: int
    top: int
    ff: int
    scale: float = 1.0
    groups: int = 1
    keep: int = 1
    shared_ff: int = 0
    #: "sigmoid": corrected scores choose, groups by the sum of their two largest,
    #: weights are the chosen plain scores' shares; "softmax": scores over all
    #: experts choose and weigh, groups by their largest
    scores: str = "sigmoid"
    act: str = "silu_glu"  # or "relu2": two matrices around the square of relu
    shared_gate: bool = True  # a sigmoid gate of one number per token

    def __post_init__(self):
        if self.scores not in ("sigmoid", "softmax") or self.act not in ("silu_glu", "relu2"):
            raise ValueError(f"unknown router {self.scores!r} or activation {self.act!r}")
        if self.experts % self.groups or not 1 <= self.keep <= self.groups \
                or not 1 <= self.top <= self.keep * (self.experts // self.groups):
            raise ValueError(f"cannot choose {self.top} of {self.experts} experts in the "
                             f"best {self.keep} of {self.groups} groups")


@dataclass(frozen=True)
class DenseSpec:
    """Ungated two-matrix feed-forward."""
    ff: int
    act: str = "xielu"  # or "gelu", the exact one


MixerSpec = Union[ParallelMixerSpec, RetentionSpec, LatentAttentionSpec, FusedMixerSpec]
MLPSpec = Union[MoESpec, GroupedMoESpec, DenseSpec]


@dataclass(frozen=True)
class LayerSpec:
    mixer: MixerSpec
    mlp: Optional[MLPSpec]


@dataclass(frozen=True)
class BigramSpec:
    """Hashed table of token pairs: row (previous * mul_prev + token * mul_cur)
    mod buckets; row ``buckets`` where there is no previous token."""
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclass(frozen=True)
class EmbeddingSpec:
    """Scaled token rows plus pair rows, normed."""
    scale: float
    bigram: BigramSpec


@dataclass
class HybridSpec:
    name: str
    hidden_size: int
    vocab_size: int
    layers: Tuple[LayerSpec, ...]
    #: (start, stop, times): these layers run ``times`` times in a row
    loop: Optional[Tuple[int, int, int]] = None
    rms_eps: float = 1e-5
    max_position: int = 131072
    arch: str = "kikalix"
    is_encoder: bool = False
    #: None: bare token rows
    embedding: Optional[EmbeddingSpec] = None
    #: taps of the causal convolution added to every mixer's input (0: none)
    input_conv: int = 0
    #: the same for every feed-forward's input
    ff_conv: int = 0
    #: each sublayer's result is scaled by a sigmoid gate of the sublayer's input
    residual_gates: bool = False
    #: what norms add to their stored weight
    norm_offset: float = 1.0
    #: beside each sublayer's input, its result is RMS normed as well
    result_norms: bool = False
    logit_scale: float = 1.0
    #: True: sublayers read the residual itself, and a layer norm with bias is
    #: taken of each sublayer's result; False: an RMS norm of each one's input
    output_norms: bool = False
    #: what goes on after a layer is a learned sum of the embedding and of every
    #: layer's result so far
    depth_average: bool = False

    def __post_init__(self):
        if self.output_norms and (self.loop or self.embedding or self.input_conv
                                  or self.ff_conv or self.residual_gates
                                  or self.result_norms):
            raise ValueError("output norms come without loops, pair embeddings, input "
                             "convolutions, residual gates and further norms")
        if self.result_norms and (self.residual_gates or self.norm_offset):
            raise ValueError("result norms come without residual gates and offsets")
        if self.depth_average and not self.output_norms:
            raise ValueError("depth averages come with output norms")
        for i, layer in enumerate(self.layers):
            j = getattr(layer.mixer, "kv_from", None)
            if j is None:
                continue
            src = self.layers[j].mixer if 0 <= j < i else None
            if not isinstance(src, LatentAttentionSpec) or src.kv_from is not None \
                    or (src.kv_rank, src.rot) != (layer.mixer.kv_rank, layer.mixer.rot):
                raise ValueError(f"layer {i}: kv_from {j} is no earlier layer with "
                                 "latents of its own, the same rank and rotation")
        if self.loop is not None:
            start, stop, times = self.loop
            if not (0 <= start < stop <= len(self.layers) and times >= 1):
                raise ValueError(f"loop {self.loop} does not fit {len(self.layers)} layers")

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    def runs(self) -> List[Tuple[int, Optional[int]]]:
        """Layer executions in order: (layer index, pass whose step vector is
        added right before it, or None). Every run owns its cache or state."""
        if self.loop is None:
            return [(i, None) for i in range(self.n_layers)]
        start, stop, times = self.loop
        out: List[Tuple[int, Optional[int]]] = [(i, None) for i in range(start)]
        for t in range(times):
            out += [(i, t if i == start else None) for i in range(start, stop)]
        return out + [(i, None) for i in range(stop, self.n_layers)]

    def param_count(self) -> int:
        w = self.hidden_size
        norm = 2 * w if self.output_norms or self.result_norms else w
        n = 2 * self.vocab_size * w + (2 * w if self.output_norms else w)
        if self.loop is not None:
            n += self.loop[2] * w
        if self.embedding is not None:
            n += (self.embedding.bigram.buckets + 2) * w
        for i, layer in enumerate(self.layers):
            n += norm * (1 if layer.mlp is None else 2)
            n += self.input_conv * w + (0 if layer.mlp is None else self.ff_conv * w)
            if self.residual_gates:
                n += (1 if layer.mlp is None else 2) * (w + 1) * w
            if self.depth_average:
                n += i + 2
            n += _mixer_params(layer.mixer, w) + _mlp_params(layer.mlp, w)
        return n


def _mixer_params(m: MixerSpec, w: int) -> int:
    if isinstance(m, FusedMixerSpec):
        return sum(_part_params(p, w) for _, p, _ in m.parts)
    if isinstance(m, RetentionSpec):
        return w * m.heads * (2 * m.dim + 3 * m.vdim)
    if isinstance(m, LatentAttentionSpec):
        rot = m.rot.dims if m.rot else 0
        q = m.heads * (m.dim + rot)
        n = m.q_rank * (w + 1 + q) if m.q_rank else w * q
        n += w * m.heads * (m.vdim + m.gate) + (m.heads if m.sink else 0)
        n += m.kv_rank * m.heads * (m.dim + m.vdim)
        return n + (m.kv_rank * (w + 1) + rot * w if m.kv_from is None else 0)
    a, r = m.left, m.right
    qkv = a.heads * a.dim + a.kv_heads * (a.dim + a.vdim)
    n = (w + 1) * qkv + w * a.heads * a.vdim
    ch = 2 * r.kv_heads * r.dim + r.heads * r.vdim
    n += ch * (w + r.conv) + w * (r.heads + r.decay_rank + r.gate_rank)
    n += r.heads * (r.dim * (r.decay_rank + 1) + r.vdim * r.gate_rank + 1)
    return n + r.vdim + w * r.heads * r.vdim


def _part_params(p: PartSpec, w: int) -> int:
    if isinstance(p, NormedAttentionSpec):
        q, k = p.heads * p.dim, p.kv_heads * p.dim
        n = w * (q + k + p.heads * p.vdim) + (2 * p.dim if p.norm == "head" else q + k)
        return n + (0 if p.shared_kv else w * p.kv_heads * p.vdim) \
            + (2 * p.heads if p.log_bias else 0)
    if isinstance(p, ConvAttentionSpec):
        ch, e = p.heads * p.dim + p.kv_heads * (p.dim + p.vdim), p.heads * p.vdim
        return ch * (w + p.conv) + w * e * (2 if p.gate else 1)
    if isinstance(p, HeadDeltaSpec):
        ch = 2 * p.kv_heads * p.dim + p.heads * p.vdim
        return ch * (w + p.conv) + 2 * p.heads * (w + 1) + p.vdim + 2 * w * p.heads * p.vdim
    return 2 * w * p.heads * (p.dim + 1) + 2 * p.heads + p.heads * p.vdim * (3 * w + 1)


def _mlp_params(f: Optional[MLPSpec], w: int) -> int:
    if f is None:
        return 0
    if isinstance(f, DenseSpec):
        return 2 * w * f.ff + (2 if f.act == "xielu" else 0)
    if isinstance(f, MoESpec):
        return f.experts * (3 * w * f.ff + w + 1)
    matrices = 3 if f.act == "silu_glu" else 2
    n = f.experts * (matrices * w * f.ff + w + (f.scores == "sigmoid"))
    return n + (w * (matrices * f.shared_ff + f.shared_gate) if f.shared_ff else 0)


AnySpec = Union[ModelSpec, HybridSpec]
_REGISTRY: Dict[str, AnySpec] = {}


def register(spec: AnySpec) -> AnySpec:
    _REGISTRY[spec.name] = spec
    return spec


# ---- checkpoint folders ------------------------------------------------------

def _kikalix_spec(name: str, cfg: dict, shapes: Dict[str, Sequence[int]]) -> HybridSpec:
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        m = entry["mixer"]
        if entry["type"] == "parallel":
            a, r = m["left"], m["right"]
            right = f"l{i}.mix.right."
            mixer: Union[ParallelMixerSpec, RetentionSpec] = ParallelMixerSpec(
                left=BiasedAttentionSpec(
                    heads=a["heads"], kv_heads=a["kv_heads"], dim=a["dim"],
                    vdim=a["vdim"], scale=float(a["scale"]),
                    window=int((a.get("mask") or {}).get("size") or 0)),
                right=DeltaRuleSpec(
                    heads=r["heads"], kv_heads=r["kv_heads"], dim=r["dim"],
                    vdim=r["vdim"], conv=r["conv"],
                    # the low-rank widths are given by the tensors alone
                    decay_rank=int(shapes[right + "a1"][0]),
                    gate_rank=int(shapes[right + "g1"][0])),
                left_scale=float(m["left_scale"]),
                right_scale=float(m["right_scale"]))
        elif entry["type"] == "retention":
            mixer = RetentionSpec(
                heads=m["heads"], dim=m["dim"], vdim=m["vdim"],
                decay=tuple(float(d) for d in m["decay"]),
                rot_dims=m["rot"]["dims"], rot_base=float(m["rot"]["base"]))
        else:
            raise ValueError(f"layer {i}: unknown mixer type {entry['type']!r}")
        ff = entry.get("mlp")
        mlp = None
        if ff is not None:
            if ff.get("kind", "moe") != "moe":
                raise ValueError(f"layer {i}: unknown feed-forward {ff['kind']!r}")
            mlp = MoESpec(experts=ff["router"]["experts"], top=ff["router"]["top"],
                          ff=ff["expert"]["ff"], limit=float(ff["expert"]["limit"]))
        layers.append(LayerSpec(mixer, mlp))
    lp = cfg.get("loop")
    return HybridSpec(
        name=name, hidden_size=cfg["width"], vocab_size=cfg["vocab"],
        layers=tuple(layers), rms_eps=float(cfg["norm"]["eps"]),
        loop=(lp["start"], lp["stop"], lp["times"]) if lp else None)


def _senotar_spec(name: str, cfg: dict, shapes: Dict[str, Sequence[int]]) -> HybridSpec:
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        if entry["type"] != "latent_attention":
            raise ValueError(f"layer {i}: unknown mixer type {entry['type']!r}")
        m, ff = entry["mixer"], entry.get("mlp")
        if ff is not None and ff.get("kind", "dense") != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward {ff['kind']!r}")
        layers.append(LayerSpec(
            LatentAttentionSpec(
                heads=m["heads"], dim=m["dim"], vdim=m["vdim"], kv_rank=m["kv_rank"],
                scale=float(m["scale"]), kv_from=m.get("kv_from")),
            DenseSpec(ff["ff"]) if ff is not None else None))
    emb = cfg["embedding"]
    bigram = emb["bigram"]
    return HybridSpec(
        name=name, arch="senotar", hidden_size=cfg["width"], vocab_size=cfg["vocab"],
        layers=tuple(layers), rms_eps=float(cfg["norm"]["eps"]), norm_offset=0.0,
        input_conv=cfg["canon"]["taps"], residual_gates=True,
        embedding=EmbeddingSpec(float(emb["scale"]), BigramSpec(
            bigram["buckets"], bigram["mul_prev"], bigram["mul_cur"])))


def _gakupel_spec(name: str, cfg: dict, shapes: Dict[str, Sequence[int]]) -> HybridSpec:
    def attention(m: dict, **kw) -> NormedAttentionSpec:
        return NormedAttentionSpec(heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
                                   vdim=m["vdim"], scale=float(m["scale"]), **kw)

    def mixer(i: int, kind: str, m: dict) -> FusedMixerSpec:
        if kind == "attention":
            rot = m["rot"]
            return FusedMixerSpec((("", attention(
                m, shared_kv=True, rot_dims=rot["dims"], rot_base=float(rot["base"])), 1.0),))
        if kind == "delta":
            return FusedMixerSpec((("", HeadDeltaSpec(
                m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]), 1.0),))
        if kind == "parallel":
            left, right = m["left"], m["right"]
            temp = left["q_temp"]
            return FusedMixerSpec((
                ("left.", attention(left, norm="whole", log_bias=True, sink=True,
                                    q_temp=(float(temp["coef"]), int(temp["every"]))),
                 float(m["left_scale"])),
                ("right.", MatrixMemorySpec(right["heads"], right["dim"], right["vdim"],
                                            float(right["gate_cap"])),
                 float(m["right_scale"]))))
        raise ValueError(f"layer {i}: unknown mixer type {kind!r}")

    def mlp(i: int, f: Optional[dict]) -> Optional[MLPSpec]:
        if f is None:
            return None
        if f["kind"] == "dense":
            return DenseSpec(f["ff"], "gelu")
        if f["kind"] == "moe":
            r = f["router"]
            groups = r.get("groups") or {"count": 1, "keep": 1}
            return GroupedMoESpec(
                experts=r["experts"], top=r["top"], ff=f["expert"]["ff"],
                scale=float(r["scale"]), groups=groups["count"], keep=groups["keep"],
                shared_ff=(f.get("shared") or {"ff": 0})["ff"])
        raise ValueError(f"layer {i}: unknown feed-forward {f['kind']!r}")

    return HybridSpec(
        name=name, arch="gakupel", hidden_size=cfg["width"], vocab_size=cfg["vocab"],
        rms_eps=float(cfg["norm"]["eps"]), norm_offset=0.0, output_norms=True,
        depth_average=True,
        layers=tuple(LayerSpec(mixer(i, e["type"], e["mixer"]), mlp(i, e.get("mlp")))
                     for i, e in enumerate(cfg["layers"])))


def _fezuzen_spec(name: str, cfg: dict, shapes: Dict[str, Sequence[int]]) -> HybridSpec:
    def rotation(r: dict) -> RotationSpec:
        y = r.get("scaling")
        return RotationSpec(r["dims"], float(r["base"]), YarnSpec(
            *(float(y[k]) for k in ("factor", "original", "fast", "slow"))) if y else None)

    def size(m: dict) -> int:
        return int((m.get("mask") or {}).get("size") or 0)

    def mixer(i: int, kind: str, m: dict) -> MixerSpec:
        if kind == "latent_attention":
            if m["rot"]["dims"] != m["rot_dim"]:
                raise ValueError(f"layer {i}: rotates {m['rot']['dims']} of {m['rot_dim']} "
                                 "dimensions")
            return LatentAttentionSpec(
                heads=m["heads"], dim=m["dim"], vdim=m["vdim"], kv_rank=m["kv_rank"],
                scale=float(m["scale"]), kv_from=m.get("kv_from"), q_rank=m["q_rank"],
                rot=rotation(m["rot"]), window=size(m), sink=False, gate=False)
        if kind == "attention":
            return FusedMixerSpec((("", ConvAttentionSpec(
                heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"],
                scale=float(m["scale"]), conv=m["conv"], rot=rotation(m["rot"]),
                value_base=float(m["rot"]["base"]), chunk=size(m), sink=True, gate=True), 1.0),))
        raise ValueError(f"layer {i}: unknown mixer type {kind!r}")

    def mlp(i: int, f: Optional[dict]) -> Optional[MLPSpec]:
        if f is None:
            return None
        if f.get("kind", "moe") != "moe":
            raise ValueError(f"layer {i}: unknown feed-forward {f['kind']!r}")
        r = f["router"]
        groups = r.get("groups") or {"count": 1, "keep": 1}
        return GroupedMoESpec(
            experts=r["experts"], top=r["top"], ff=f["expert"]["ff"], groups=groups["count"],
            keep=groups["keep"], shared_ff=(f.get("shared") or {"ff": 0})["ff"],
            scores="softmax", act="relu2", shared_gate=False)

    taps = cfg["canon"]["taps"]
    return HybridSpec(
        name=name, arch="fezuzen", hidden_size=cfg["width"], vocab_size=cfg["vocab"],
        rms_eps=float(cfg["norm"]["eps"]), norm_offset=0.0, result_norms=True,
        input_conv=taps, ff_conv=taps, logit_scale=float(cfg["logit_scale"]),
        layers=tuple(LayerSpec(mixer(i, e["type"], e["mixer"]), mlp(i, e.get("mlp")))
                     for i, e in enumerate(cfg["layers"])))


#: config.json "architecture" -> reader(name, config, tensor shapes)
_CONFIG_READERS = {"Kikalix": _kikalix_spec, "Senotar": _senotar_spec,
                   "Gakupel": _gakupel_spec, "Fezuzen": _fezuzen_spec}


def is_checkpoint_dir(path: str) -> bool:
    return os.path.isfile(os.path.join(path, "config.json"))


def spec_from_checkpoint(path: str) -> AnySpec:
    """Spec of a checkpoint folder (config.json beside *.safetensors)."""
    from .loader import tensor_shapes

    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    arch = cfg.get("architecture")
    reader = _CONFIG_READERS.get(arch)
    if reader is None:
        raise KeyError(f"unknown architecture {arch!r} in {path}/config.json; "
                       f"known: {sorted(_CONFIG_READERS)}")
    name = os.path.basename(os.path.normpath(path)) or path
    return reader(name, cfg, tensor_shapes(path))


def get_spec(name: str) -> AnySpec:
    """A registered spec by name, or the spec of a checkpoint folder."""
    if name not in _REGISTRY and is_checkpoint_dir(name):
        return spec_from_checkpoint(name)
    try:
        return _REGISTRY[name]
    except KeyError:
        raise KeyError(f"unknown model spec '{name}'; known: {sorted(_REGISTRY)}") from None


# ---- presets -------------------------------------

register(ModelSpec(  # BASELINE config 2/5 agent model
    name="llama3-8b", hidden_size=4096, n_layers=32, n_heads=32, n_kv_heads=8,
    head_dim=128, intermediate_size=14336, vocab_size=128256,
))
register(ModelSpec(
    name="llama3-70b", hidden_size=8192, n_layers=80, n_heads=64, n_kv_heads=8,
    head_dim=128, intermediate_size=28672, vocab_size=128256,
))
register(ModelSpec(
    name="llama3.2-1b", hidden_size=2048, n_layers=16, n_heads=32, n_kv_heads=8,
    head_dim=64, intermediate_size=8192, vocab_size=128256, tie_embeddings=True,
))
register(ModelSpec(  # BASELINE config 4 (MoE tool-calling agent)
    name="mixtral-8x7b", hidden_size=4096, n_layers=32, n_heads=32, n_kv_heads=8,
    head_dim=128, intermediate_size=14336, vocab_size=32000, rope_theta=1e6,
    n_experts=8, experts_per_token=2,
))
register(ModelSpec(  # Qwen2/2.5-7B: llama arch + QKV bias, 1e6 rope, 152k vocab
    name="qwen2-7b", hidden_size=3584, n_layers=28, n_heads=28, n_kv_heads=4,
    head_dim=128, intermediate_size=18944, vocab_size=152064, rope_theta=1e6,
    max_position=32768, rms_eps=1e-6, qkv_bias=True,
))
register(ModelSpec(
    name="qwen2-72b", hidden_size=8192, n_layers=80, n_heads=64, n_kv_heads=8,
    head_dim=128, intermediate_size=29568, vocab_size=152064, rope_theta=1e6,
    max_position=32768, rms_eps=1e-6, qkv_bias=True,
))
register(ModelSpec(  # BGE-base-style embedding encoder (RAG path)
    name="bge-base", hidden_size=768, n_layers=12, n_heads=12, n_kv_heads=12,
    head_dim=64, intermediate_size=3072, vocab_size=30522, is_encoder=True,
    max_position=512, rms_eps=1e-12,
))
# tiny configs for CPU tests / plumbing validation
register(ModelSpec(
    name="tiny-llama", hidden_size=64, n_layers=2, n_heads=4, n_kv_heads=2,
    head_dim=16, intermediate_size=128, vocab_size=512, max_position=2048,
    tie_embeddings=True,
))
register(ModelSpec(  # Qwen2-shaped tiny config (qkv_bias path on CPU)
    name="tiny-qwen", hidden_size=64, n_layers=2, n_heads=4, n_kv_heads=2,
    head_dim=16, intermediate_size=128, vocab_size=512, max_position=2048,
    rope_theta=1e6, qkv_bias=True, tie_embeddings=True,
))
register(ModelSpec(
    name="tiny-moe", hidden_size=64, n_layers=2, n_heads=4, n_kv_heads=2,
    head_dim=16, intermediate_size=96, vocab_size=512, max_position=2048,
    n_experts=4, experts_per_token=2, tie_embeddings=True,
))
register(ModelSpec(
    name="tiny-encoder", hidden_size=64, n_layers=2, n_heads=4, n_kv_heads=4,
    head_dim=16, intermediate_size=128, vocab_size=512, max_position=512,
    is_encoder=True,
))
register(ModelSpec(  # GPU smoke/test model: real head_dim for the HIP kernels
    name="smoke-llama", hidden_size=512, n_layers=4, n_heads=4, n_kv_heads=2,
    head_dim=128, intermediate_size=1024, vocab_size=1024, max_position=8192,
    tie_embeddings=True,
))
register(ModelSpec(  # GPU long-context smoke: 64k positions, tiny layers
    name="smoke-llama-64k", hidden_size=512, n_layers=4, n_heads=4,
    n_kv_heads=2, head_dim=128, intermediate_size=1024, vocab_size=1024,
    max_position=65536, tie_embeddings=True,
))
register(ModelSpec(  # GPU Qwen2-shaped smoke: qkv_bias on the HIP path
    name="smoke-qwen", hidden_size=512, n_layers=4, n_heads=4, n_kv_heads=2,
    head_dim=128, intermediate_size=1024, vocab_size=1024, max_position=8192,
    rope_theta=1e6, qkv_bias=True, tie_embeddings=True,
))
register(ModelSpec(  # GPU MoE smoke: real head_dim for the HIP kernels
    name="smoke-moe", hidden_size=512, n_layers=4, n_heads=4, n_kv_heads=2,
    head_dim=128, intermediate_size=768, vocab_size=1024, max_position=8192,
    n_experts=4, experts_per_token=2, tie_embeddings=True,
))

# ---- Kikalix presets ---------------------------------------------------------

def kikalix_layers(pattern: str, *, heads: int, kv_heads: int, dim: int, vdim: int,
                   window: int, d_heads: int, d_kv_heads: int, d_dim: int,
                   d_vdim: int, rank: int, r_heads: int, r_dim: int, r_vdim: int,
                   experts: int, top: int, ff: int, conv: int = 4,
                   limit: float = 7.0, rot_base: float = 1e4) -> Tuple[LayerSpec, ...]:
    """Layers of one size from a pattern: 'p' parallel, 'r' retention."""
    moe = MoESpec(experts=experts, top=top, ff=ff, limit=limit)
    par = ParallelMixerSpec(
        left=BiasedAttentionSpec(heads, kv_heads, dim, vdim, dim ** -0.5, window),
        right=DeltaRuleSpec(d_heads, d_kv_heads, d_dim, d_vdim, conv, rank, rank),
        left_scale=0.5, right_scale=0.5)
    ret = RetentionSpec(r_heads, r_dim, r_vdim,
                        tuple(1.0 - 2.0 ** (-5 - 3.0 * h / max(r_heads - 1, 1))
                              for h in range(r_heads)), r_dim, rot_base)
    return tuple(LayerSpec({"p": par, "r": ret}[c], moe) for c in pattern)


register(HybridSpec(  # CPU plumbing size
    name="tiny-kikalix", hidden_size=64, vocab_size=512, max_position=2048,
    loop=(1, 3, 2), layers=kikalix_layers(
        "prp", heads=4, kv_heads=2, dim=16, vdim=24, window=20, d_heads=4,
        d_kv_heads=2, d_dim=16, d_vdim=8, rank=6, r_heads=3, r_dim=16, r_vdim=12,
        experts=5, top=2, ff=40),
))
register(HybridSpec(  # GPU smoke size: the matrix-core kernels' head widths
    name="smoke-kikalix", hidden_size=512, vocab_size=1024, max_position=8192,
    loop=(0, 2, 2), layers=kikalix_layers(
        "rpp", heads=8, kv_heads=2, dim=128, vdim=128, window=300, d_heads=4,
        d_kv_heads=2, d_dim=128, d_vdim=128, rank=32, r_heads=4, r_dim=128,
        r_vdim=128, experts=8, top=2, ff=256),
))
register(HybridSpec(  # layer sizes of a 7B-class decoder, 8 experts like mixtral-8x7b
    name="kikalix-8x7b", hidden_size=4096, vocab_size=32000,
    layers=kikalix_layers(
        "ppprpppr" * 4, heads=32, kv_heads=8, dim=128, vdim=128, window=1024,
        d_heads=16, d_kv_heads=16, d_dim=128, d_vdim=128, rank=128, r_heads=16,
        r_dim=256, r_vdim=256, experts=8, top=2, ff=14336),
))

# ---- Senotar presets ---------------------------------------------------------

def senotar_spec(name: str, pattern: str, *, width: int, vocab: int, heads: int, dim: int,
                 vdim: int, kv_rank: int, ff: int, taps: int = 4, buckets: int = 65521,
                 max_position: int = 131072) -> HybridSpec:
    """Layers of one size from a pattern: 'o' has latents of its own, 's' reads
    the last 'o' layer's; upper case: without a feed-forward."""
    layers, own = [], None
    for i, c in enumerate(pattern):
        if c in "oO":
            own = i
        mixer = LatentAttentionSpec(heads, dim, vdim, kv_rank, dim ** -0.5,
                                    None if c in "oO" else own)
        layers.append(LayerSpec(mixer, None if c.isupper() else DenseSpec(ff)))
    return HybridSpec(
        name=name, arch="senotar", hidden_size=width, vocab_size=vocab, layers=tuple(layers),
        max_position=max_position, input_conv=taps, residual_gates=True, norm_offset=0.0,
        embedding=EmbeddingSpec(width ** 0.5, BigramSpec(buckets, 31, 17)))


register(senotar_spec(  # CPU plumbing size
    "tiny-senotar", "oOss", width=64, vocab=512, heads=3, dim=16, vdim=24, kv_rank=20,
    ff=96, taps=3, buckets=97, max_position=2048))
register(senotar_spec(  # GPU smoke size
    "smoke-senotar", "ooss", width=512, vocab=1024, heads=8, dim=64, vdim=64, kv_rank=256,
    ff=1024, buckets=509, max_position=8192))
register(senotar_spec(  # layer sizes of a 7B-class decoder
    "senotar-7b", "o" * 16 + "s" * 16, width=4096, vocab=32000, heads=32, dim=128,
    vdim=128, kv_rank=512, ff=14336))

# ---- Gakupel presets ---------------------------------------------------------

def gakupel_spec(name: str, pattern: str, *, width: int, vocab: int, heads: int,
                 kv_heads: int, dim: int, l_dim: int, l_vdim: int, d_heads: int,
                 d_kv_heads: int, d_dim: int, d_vdim: int, m_heads: int, m_dim: int,
                 m_vdim: int, ff: int, experts: int, top: int, expert_ff: int,
                 shared_ff: int, groups: int = 4, keep: int = 2, conv: int = 4,
                 rot_dims: int = 0, max_position: int = 131072) -> HybridSpec:
    """Layers of one size from a pattern: 'a' attention, 'd' delta rule, 'p'
    attention beside a matrix memory; upper case: dense instead of routed."""
    mixers = {
        "a": FusedMixerSpec((("", NormedAttentionSpec(
            heads, kv_heads, dim, dim, dim ** -0.5, rot_dims=rot_dims or dim,
            shared_kv=True), 1.0),)),
        "d": FusedMixerSpec((("", HeadDeltaSpec(d_heads, d_kv_heads, d_dim, d_vdim, conv),
                              1.0),)),
        "p": FusedMixerSpec((
            ("left.", NormedAttentionSpec(
                heads, kv_heads, l_dim, l_vdim, l_dim ** -0.5, norm="whole",
                q_temp=(0.2, 1024), log_bias=True, sink=True), 0.7),
            ("right.", MatrixMemorySpec(m_heads, m_dim, m_vdim, 15.0), 0.7)))}
    moe = GroupedMoESpec(experts, top, expert_ff, 2.0, groups, keep, shared_ff)
    return HybridSpec(
        name=name, arch="gakupel", hidden_size=width, vocab_size=vocab,
        max_position=max_position, norm_offset=0.0, output_norms=True, depth_average=True,
        layers=tuple(LayerSpec(mixers[c.lower()], DenseSpec(ff, "gelu") if c.isupper() else moe)
                     for c in pattern))


register(gakupel_spec(  # CPU plumbing size
    "tiny-gakupel", "Pad", width=64, vocab=512, heads=4, kv_heads=2, dim=16,
    l_dim=12, l_vdim=20, d_heads=4, d_kv_heads=2, d_dim=16, d_vdim=8, m_heads=3, m_dim=8,
    m_vdim=12, ff=96, experts=6, top=2, expert_ff=24, shared_ff=40, groups=3, rot_dims=8,
    max_position=2048))
register(gakupel_spec(  # GPU smoke size: the matrix-core kernels' head widths
    "smoke-gakupel", "paDp", width=512, vocab=1024, heads=8, kv_heads=2, dim=64,
    l_dim=128, l_vdim=64, d_heads=4, d_kv_heads=2, d_dim=128, d_vdim=128, m_heads=4,
    m_dim=64, m_vdim=128, ff=1024, experts=16, top=2, expert_ff=128, shared_ff=256,
    max_position=8192))
register(gakupel_spec(  # layer sizes of a 7B-class decoder, 8 experts like mixtral-8x7b
    "gakupel-8x7b", "pdaPpdap" * 4, width=4096, vocab=32000, heads=32, kv_heads=8, dim=128,
    l_dim=128, l_vdim=128, d_heads=16, d_kv_heads=16, d_dim=128, d_vdim=256,
    m_heads=16, m_dim=128, m_vdim=256, ff=14336, experts=8, top=2, expert_ff=14336,
    shared_ff=14336, groups=4, keep=2))

# ---- Fezuzen presets ---------------------------------------------------------

def fezuzen_spec(name: str, pattern: str, *, width: int, vocab: int, heads: int, dim: int,
                 rot_dim: int, vdim: int, kv_rank: int, q_rank: int, window: int,
                 a_heads: int, kv_heads: int, a_dim: int, a_vdim: int, chunk: int,
                 experts: int, top: int, expert_ff: int, shared_ff: int, groups: int = 4,
                 keep: int = 2, taps: int = 4, conv: int = 4, base: float = 5e5,
                 max_position: int = 131072) -> HybridSpec:
    """Layers of one size from a pattern: 'o' latent attention with latents of its
    own, 's' reading the last 'o' layer's, 'a' convolved attention; upper case:
    without a feed-forward."""
    yarn = YarnSpec(4.0, max_position / 4, 32.0, 1.0)
    layers, own = [], None
    moe = GroupedMoESpec(experts, top, expert_ff, 1.0, groups, keep, shared_ff,
                         "softmax", "relu2", False)
    for i, c in enumerate(pattern):
        if c in "oO":
            own = i
        if c in "aA":
            mixer: MixerSpec = FusedMixerSpec((("", ConvAttentionSpec(
                a_heads, kv_heads, a_dim, a_vdim, a_dim ** -0.5, conv,
                RotationSpec(a_dim, base), value_base=base, chunk=chunk, sink=True,
                gate=True), 1.0),))
        else:
            mixer = LatentAttentionSpec(
                heads, dim, vdim, kv_rank, (dim + rot_dim) ** -0.5,
                None if c in "oO" else own, q_rank, RotationSpec(rot_dim, base, yarn), window,
                sink=False, gate=False)
        layers.append(LayerSpec(mixer, None if c.isupper() else moe))
    return HybridSpec(
        name=name, arch="fezuzen", hidden_size=width, vocab_size=vocab, layers=tuple(layers),
        max_position=max_position, norm_offset=0.0, result_norms=True, input_conv=taps,
        ff_conv=taps, logit_scale=0.25)


register(fezuzen_spec(  # CPU plumbing size
    "tiny-fezuzen", "oaSo", width=64, vocab=512, heads=3, dim=16, rot_dim=8, vdim=24,
    kv_rank=20, q_rank=28, window=30, a_heads=4, kv_heads=2, a_dim=16, a_vdim=12, chunk=24,
    experts=6, top=2, expert_ff=24, shared_ff=40, groups=3, taps=3, max_position=2048))
register(fezuzen_spec(  # GPU smoke size: the matrix-core kernels' head widths
    "smoke-fezuzen", "oaso", width=512, vocab=1024, heads=8, dim=128, rot_dim=64, vdim=128,
    kv_rank=256, q_rank=384, window=300, a_heads=8, kv_heads=2, a_dim=128, a_vdim=64,
    chunk=200, experts=16, top=2, expert_ff=128, shared_ff=256, max_position=8192))
register(fezuzen_spec(  # layer sizes of a 2048 wide decoder, 64 experts
    "fezuzen-13b", "oasa" * 8, width=2048, vocab=32000, heads=16, dim=128, rot_dim=64,
    vdim=128, kv_rank=512, q_rank=1536, window=4096, a_heads=16, kv_heads=4, a_dim=128,
    a_vdim=128, chunk=8192, experts=64, top=6, expert_ff=1408, shared_ff=2816, groups=8,
    keep=3))
