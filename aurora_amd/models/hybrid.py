"""Layer-listed decoders (Kikalix, Senotar, Gakupel, Fezuzen): mixers and
feed-forwards chosen layer by layer, with a span of layers that may run several
times.

Same engine shape as the other decoders: packed varlen tokens, paged KV and
per-step metadata. Two things differ. The residual stream is one fp32 tensor
that every norm kernel updates in place (the preceding sub-layer's output, or
the weighted expert rows, and the pass vector are added by the kernel that
norms; where norms are taken of the sub-layers' outputs, so are the normed
output and the average over the depth). And every layer RUN, not layer, owns a
paged cache or recurrent state; a mixer may instead read an earlier layer's cache.
Beside the mixers', state is what input convolutions and a pair embedding remember
of the last tokens.
"""
from __future__ import annotations

from typing import Dict, List, Tuple

import torch
import torch.nn as nn

from .. import ops
from ..parallel import dist as pdist
from .config import (
    DenseSpec,
    FusedMixerSpec,
    GroupedMoESpec,
    HybridSpec,
    LatentAttentionSpec,
    ParallelMixerSpec,
)
from .llama import AttnMetadata
from .mixers import (
    DenseGeluMLP,
    DenseXieluMLP,
    FusedMixer,
    GroupedExperts,
    LatentAttention,
    ParallelMixer,
    RetentionMixer,
    RoutedGLU,
    _param,
)


class HybridLayer(nn.Module):
    def __init__(self, spec: HybridSpec, i: int, dtype, rotations: dict):
        super().__init__()
        s = spec.layers[i]
        w = spec.hidden_size
        self.norm1 = _param(w, dtype=torch.float32)
        self.norm1_bias = _param(w, dtype=torch.float32) if spec.output_norms else None
        self.norm2_bias = None
        # weights of the embedding's and every layer's result in what goes on
        self.depth = _param(i + 2, dtype=torch.float32) if spec.depth_average else None
        if isinstance(s.mixer, FusedMixerSpec):
            self.mixer: nn.Module = FusedMixer(s.mixer, w, spec.rms_eps, dtype,
                                               spec.max_position, rotations)
        elif isinstance(s.mixer, ParallelMixerSpec):
            self.mixer = ParallelMixer(s.mixer, w, spec.rms_eps, dtype)
        elif isinstance(s.mixer, LatentAttentionSpec):
            self.mixer = LatentAttention(s.mixer, w, spec.rms_eps, dtype,
                                         spec.max_position, rotations)
        else:
            m = s.mixer
            key = (m.rot_dims, m.rot_base)
            if key not in rotations:  # one table for all layers that share it
                rotations[key] = ops.torch_ref.rope_cos_sin_cache(
                    m.rot_dims, spec.max_position, m.rot_base)
            self.mixer = RetentionMixer(m, w, spec.rms_eps, dtype, rotations[key])
        # convolution of the mixer's input, residual gate of its output
        self.conv = _param(spec.input_conv, w, dtype=torch.float32) \
            if spec.input_conv else None
        self.ff_conv = _param(spec.ff_conv, w, dtype=torch.float32) \
            if spec.ff_conv and s.mlp is not None else None
        # norms of the sublayers' results
        self.post1 = _param(w, dtype=torch.float32) if spec.result_norms else None
        self.post2 = _param(w, dtype=torch.float32) \
            if spec.result_norms and s.mlp is not None else None
        self.gate = _param(w, w, dtype=dtype) if spec.residual_gates else None
        self.gate_bias = _param(w, dtype=torch.float32) if spec.residual_gates else None
        if s.mlp is None:
            self.mlp = None
            return
        self.norm2 = _param(w, dtype=torch.float32)
        if spec.output_norms:
            self.norm2_bias = _param(w, dtype=torch.float32)
        if isinstance(s.mlp, GroupedMoESpec) and s.mlp.shared_gate and s.mlp.shared_ff \
                and not spec.output_norms:
            raise ValueError("a shared expert's gate needs output norms")
        if isinstance(s.mlp, GroupedMoESpec) or getattr(s.mlp, "act", None) == "gelu":
            if spec.residual_gates:
                raise ValueError(f"no residual gates around a {type(s.mlp).__name__}")
            self.mlp = GroupedExperts(s.mlp, w, dtype) if isinstance(s.mlp, GroupedMoESpec) \
                else DenseGeluMLP(s.mlp, w, dtype)
        elif isinstance(s.mlp, DenseSpec):
            self.mlp = DenseXieluMLP(s.mlp, w, dtype, spec.residual_gates)
        elif spec.residual_gates:
            raise ValueError("routed experts have no residual gate")
        else:
            self.mlp = RoutedGLU(s.mlp, w, dtype)

    def state_layout(self, dtype) -> List[tuple]:
        """The input convolutions' last inputs, if there are any, then the mixer's."""
        own = []
        for conv in (self.conv, self.ff_conv):
            if conv is not None:
                taps, w = conv.shape
                own.append((((taps - 1, w), dtype),))
        return own + self.mixer.state_layout(dtype)


class HybridForCausalLM(nn.Module):
    def __init__(self, spec: HybridSpec, dtype=torch.bfloat16, device=None):
        super().__init__()
        if pdist.tp_world_size() > 1:
            raise NotImplementedError(
                f"{spec.name}: layer-listed decoders run with tp_size=1 "
                "(shard requests over GPUs instead)")
        self.spec = spec
        self.dtype = dtype
        with torch.device(device or "cpu"):
            self.embed = nn.Embedding(spec.vocab_size, spec.hidden_size, dtype=dtype)
            self.embed.weight.requires_grad_(False)
            rotations: dict = {}
            self.layers = nn.ModuleList(
                [HybridLayer(spec, i, dtype, rotations) for i in range(spec.n_layers)])
            self.final_norm = _param(spec.hidden_size, dtype=torch.float32)
            self.final_norm_bias = _param(spec.hidden_size, dtype=torch.float32) \
                if spec.output_norms else None
            self.lm_head = _param(spec.vocab_size, spec.hidden_size, dtype=dtype)
            # fp32 and not a scalar, so that the product is fp32 too
            self.register_buffer("logit_scale", torch.tensor([spec.logit_scale]).float()
                                 if spec.logit_scale != 1.0 else None, persistent=False)
            self.loop_step = _param(spec.loop[2], spec.hidden_size,
                                    dtype=torch.float32) if spec.loop else None
            if spec.embedding is not None:
                self.pairs = _param(spec.embedding.bigram.buckets + 1, spec.hidden_size,
                                    dtype=dtype)
                self.embed_norm = _param(spec.hidden_size, dtype=torch.float32)
        # run -> its paged caches and state entries, in kv_layout / state_layout
        # order
        self._runs: List[tuple] = []
        last_kv: Dict[int, slice] = {}
        n_kv, n_state = 0, len(self._embed_state())
        for i, step in spec.runs():
            layer = self.layers[i]
            a = len(layer.mixer.kv_layout(dtype, "cpu"))
            b = len(layer.state_layout(dtype))
            source = getattr(spec.layers[i].mixer, "kv_from", None)
            last_kv[i] = slice(n_kv, n_kv + a) if source is None else last_kv[source]
            self._runs.append((i, step, last_kv[i], slice(n_state, n_state + b)))
            n_kv, n_state = n_kv + a, n_state + b

    def kv_layout(self) -> List[Tuple[int, int, int]]:
        dev = self.embed.weight.device
        return [e for i, _ in self.spec.runs()
                for e in self.layers[i].mixer.kv_layout(self.dtype, dev)]

    def _embed_state(self) -> List[tuple]:
        # a pair embedding remembers the last token
        return [(((1,), torch.int32),)] if self.spec.embedding is not None else []

    def state_layout(self) -> List[tuple]:
        """The embedding's state, then per run with a state the (shape, dtype) of
        each of its tensors' slots."""
        return self._embed_state() + [
            e for i, _ in self.spec.runs() for e in self.layers[i].state_layout(self.dtype)]

    def _embed(self, input_ids, meta, segments) -> torch.Tensor:
        e = self.spec.embedding
        if e is None:
            return self.embed(input_ids).float()
        return ops.embed_pairs(
            input_ids, self.embed.weight, e.scale, self.pairs, e.bigram.mul_prev,
            e.bigram.mul_cur, self.embed_norm, self.spec.rms_eps, meta.states[0][0],
            segments)

    @torch.inference_mode()
    def forward(self, input_ids: torch.Tensor, kv_caches, meta: AttnMetadata,
                trail=None) -> torch.Tensor:
        """Normed hidden states [T, H]; ``trail``, if a list, receives the
        residual stream after every layer run."""
        segments = meta.segments(input_ids.shape[0])
        states = meta.states or []  # a model need not have any
        if self.spec.output_norms:
            return self._forward_output_normed(input_ids, kv_caches, meta, segments, states, trail)
        x = self._embed(input_ids, meta, segments)
        norm = {"eps": self.spec.rms_eps, "offset": self.spec.norm_offset,
                "dtype": self.dtype}
        add: Dict[str, object] = {}  # what the next norm adds to the residual

        def read(weight, conv, state):
            """The sublayer's normed input, what it reads, and the mixer's state."""
            if conv is None:
                h = ops.residual_rmsnorm(x, weight, **norm, **add)
                return h, h, state
            h, u = ops.residual_rmsnorm_conv(x, weight, conv_w=conv, ring=state[0][0],
                                             segments=segments, **norm, **add)
            return h, u, state[1:]

        for i, step, kv, st in self._runs:
            layer = self.layers[i]
            state = states[st]
            if step is not None:
                add["step"] = self.loop_step[step]
            h, u, state = read(layer.norm1, layer.conv, state)
            ff_state, state = (state[:1], state[1:]) if layer.ff_conv is not None else ([], state)
            add = {"delta": layer.mixer(u, meta, segments, kv_caches[kv], state)}
            if layer.gate is not None:
                add["gate"] = (ops.linear(h, layer.gate), layer.gate_bias)
            if layer.post1 is not None:
                add["post"] = layer.post1
            if layer.mlp is not None:
                h, u, _ = read(layer.norm2, layer.ff_conv, ff_state)
                add = layer.mlp(u)
                if layer.post2 is not None:
                    add["post"] = layer.post2
            if trail is not None:
                y = x.clone()
                ops.residual_rmsnorm(y, layer.norm1, **norm, **add)
                trail.append(y)
        return ops.residual_rmsnorm(x, self.final_norm, **norm, **add)

    def _forward_output_normed(self, input_ids, kv_caches, meta, segments, states, trail):
        """Sublayers read the residual itself; one kernel per sublayer norms its
        result, adds it, and after a layer takes the average over the depth, after
        the last one the final norm as well."""
        T, n = input_ids.shape[0], len(self._runs)
        h = self.embed(input_ids)
        if self.spec.depth_average:  # the embedding's and the layers' results
            kept = torch.empty(n, T, h.shape[1], dtype=torch.float32, device=h.device)
            src = kept[0].copy_(h)
        else:
            kept, src = None, h.float()
        x = torch.empty_like(src)
        norm = {"eps": self.spec.rms_eps, "dtype": self.dtype}
        for run, (i, _, kv, st) in enumerate(self._runs):
            layer = self.layers[i]
            last = {} if kept is None else {"depth": (kept, layer.depth)}
            if run == n - 1:
                last["final"] = (self.final_norm, self.final_norm_bias)
            y = layer.mixer(h, meta, segments, kv_caches[kv], states[st])
            h = ops.output_norm(src, x, layer.norm1, layer.norm1_bias, delta=y, **norm,
                                **(last if layer.mlp is None else {}))
            if layer.mlp is not None:
                h = ops.output_norm(x, x, layer.norm2, layer.norm2_bias, **layer.mlp(h),
                                    **norm, **last)
            src = x
            if trail is not None:
                trail.append(x.clone())
        return h

    @torch.inference_mode()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        logits = ops.linear(hidden, self.lm_head)
        return logits.float() if self.logit_scale is None else logits * self.logit_scale

    @torch.inference_mode()
    def load_tensors(self, get) -> None:
        """Fill every weight from ``get(name) -> tensor``."""
        for name, t in self._plain_tensors().items():
            t.copy_(get(name))
        for i, layer in enumerate(self.layers):
            layer.mixer.load(lambda n, i=i: get(f"l{i}.mix.{n}"))
            if layer.mlp is None:
                continue
            read = [lambda n, i=i: get(f"l{i}.mlp.{n}")]
            if layer.gate is not None:
                read.append(lambda n, i=i: get(f"l{i}.rg2{n}"))
            layer.mlp.load(*read)

    def _plain_tensors(self) -> Dict[str, torch.Tensor]:
        """Weights held as they are stored (or views of them), by name."""
        out = {"embed": self.embed.weight.data, "final.norm": self.final_norm.data,
               "head": self.lm_head.data}
        if self.final_norm_bias is not None:
            out["final.norm.b"] = self.final_norm_bias.data
        if self.loop_step is not None:
            out["loop.step"] = self.loop_step.data
        if self.spec.embedding is not None:
            out["bigram"], out["embed.norm"] = self.pairs.data, self.embed_norm.data
        for i, layer in enumerate(self.layers):
            out[f"l{i}.norm1"] = layer.norm1.data
            if layer.mlp is not None:
                out[f"l{i}.norm2"] = layer.norm2.data
            for name, t in (("norm1.b", layer.norm1_bias), ("norm2.b", layer.norm2_bias),
                            ("dwa", layer.depth)):
                if t is not None:
                    out[f"l{i}.{name}"] = t.data
            for name, t in (("norm1b", layer.post1), ("norm2b", layer.post2)):
                if t is not None:
                    out[f"l{i}.{name}"] = t.data
            for name, t in (("canon1", layer.conv), ("canon2", layer.ff_conv)):
                if t is not None:
                    out[f"l{i}.{name}"] = t.data.t()
            if layer.gate is not None:
                out[f"l{i}.rg1"], out[f"l{i}.rg1.b"] = layer.gate.data, layer.gate_bias.data
        return out

    def named_tensors(self) -> Dict[str, torch.Tensor]:
        """Inverse of ``load_tensors``."""
        out = self._plain_tensors()
        for i, layer in enumerate(self.layers):
            parts = [(f"l{i}.mix.", layer.mixer.tensors())]
            if layer.mlp is not None:
                parts.append((f"l{i}.mlp.", layer.mlp.tensors()))
                if layer.gate is not None:
                    parts.append((f"l{i}.rg2", layer.mlp.gate_tensors()))
            for tag, tensors in parts:
                out.update({tag + n: t.data for n, t in tensors.items()})
        return out

    @torch.inference_mode()
    def init_random(self, seed: int = 0) -> None:
        """Random weights; small tensors come from a CPU generator so that CPU
        and GPU instances of one spec agree, big ones are drawn on the device."""
        gen = torch.Generator(device="cpu").manual_seed(seed)
        dev = self.embed.weight.device
        dev_gen = None if dev.type == "cpu" else \
            torch.Generator(device=dev).manual_seed(seed)

        def randn(shape):
            n = 1
            for s in shape:
                n *= s
            if dev_gen is not None and n > (1 << 24):
                return torch.randn(shape, generator=dev_gen, device=dev)
            return torch.randn(shape, generator=gen).to(dev)

        w = self.spec.hidden_size

        def norm_weight():  # norms scale by about one
            return 1.0 - self.spec.norm_offset + randn((w,)) * 0.1

        self.embed.weight.copy_(randn(self.embed.weight.shape))
        self.lm_head.copy_(randn(self.lm_head.shape) * w ** -0.5)
        self.final_norm.copy_(norm_weight())
        if self.loop_step is not None:
            self.loop_step.copy_(randn(self.loop_step.shape) * 0.1)
        if self.spec.embedding is not None:
            self.pairs.copy_(randn(self.pairs.shape))
            self.embed_norm.copy_(norm_weight())
        for bias in [self.final_norm_bias] + [b for layer in self.layers for b in
                                              (layer.norm1_bias, layer.norm2_bias)]:
            if bias is not None:
                bias.copy_(randn((w,)) * 0.1)
        for layer in self.layers:
            if layer.depth is not None:  # mostly the last, something of all
                layer.depth.copy_(randn(tuple(layer.depth.shape)) * 0.1)
                layer.depth[-1] += 1.0
            layer.norm1.copy_(norm_weight())
            layer.mixer.init_random(randn)
            for conv in (layer.conv, layer.ff_conv):
                if conv is not None:
                    conv.copy_(randn(conv.shape) * 0.3)
            for post in (layer.post1, layer.post2):
                if post is not None:
                    post.copy_(norm_weight())
            if layer.gate is not None:
                layer.gate.copy_(randn((w, w)) * w ** -0.5)
                layer.gate_bias.copy_(randn((w,)))
            if layer.mlp is not None:
                layer.norm2.copy_(norm_weight())
                layer.mlp.init_random(randn)
