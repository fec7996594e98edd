"""Architecture -> model class and weight loader.

The engine builds every decoder through ``build_model``; a new architecture
adds one line to ``_ARCHS`` (and its config.json reader to models.config).
"""
from __future__ import annotations

from typing import Optional

from .config import AnySpec


def _llama(spec, dtype, device):
    from .llama import LlamaForCausalLM
    return LlamaForCausalLM(spec, dtype=dtype, device=device)


def _load_llama(model, path):
    from .loader import load_llama_safetensors
    return load_llama_safetensors(model, path)


def _hybrid(spec, dtype, device):
    from .hybrid import HybridForCausalLM
    return HybridForCausalLM(spec, dtype=dtype, device=device)


def _load_named(model, path):
    from .loader import load_named_safetensors
    return load_named_safetensors(model, path)


_ARCHS = {
    "llama": (_llama, _load_llama),
    "kikalix": (_hybrid, _load_named),
    "senotar": (_hybrid, _load_named),
    "gakupel": (_hybrid, _load_named),
    "fezuzen": (_hybrid, _load_named),
}


def build_model(spec: AnySpec, dtype, device, checkpoint: Optional[str] = None,
                seed: int = 0):
    """The model of ``spec`` with the checkpoint's weights, or random ones."""
    make, load = _ARCHS[spec.arch]
    model = make(spec, dtype, device)
    if checkpoint:
        load(model, checkpoint)
    else:
        model.init_random(seed)
    return model.eval()
