"""Python host-side mirror of puppygrad's GPT-2 model/runtime API over the HIP C ABI (what every
architecture shares is in model.py).

Names, argument meaning and error behaviour follow the reference
(src/models/gpt2/rust.rs, src/models/autoregressive.rs, src/models/generation.rs)
so tests read like the reference's own: `Gpt2Model.new(config, weights)`,
`model.new_kv_cache()`, `model.prefill(ids, cache)`, `model.forward_one(id, cache)`,
`model.select_next_token(logits)`, `generate(model, ids, max_new, on_token)`.
All compute happens inside libpuppygrad_hip.so.
"""
from __future__ import annotations

import ctypes as C
from dataclasses import dataclass
from typing import List, Optional

import numpy as np

from . import _lib
from .model import (DeviceLogits, GenerationStats, Gpt2Error, Gpt2HipConfig, Gpt2OperationProfile, Gpt2Output,
                    KvCache, LogitsSampler, Model, TensorStore, TextGenerationConfig, _check, argmax_logits,
                    generate)

GPT2_EOS_TOKEN_ID = 50_256  # src/models/gpt2/options.rs:8


@dataclass
class Gpt2Config:
    """Gpt2Config (src/models/gpt2/rust.rs:30-58)."""
    vocab_size: int
    n_positions: int
    n_embd: int
    n_layer: int
    n_head: int
    n_inner: Optional[int] = None
    layer_norm_epsilon: float = 1e-5

    def __post_init__(self):
        if self.n_inner is None:
            self.n_inner = 4 * self.n_embd

    def head_dim(self) -> int:
        return self.n_embd // self.n_head

    def to_c(self) -> _lib.pg_gpt2_config:
        return _lib.pg_gpt2_config(self.vocab_size, self.n_positions, self.n_embd, self.n_layer,
                                   self.n_head, self.n_inner, self.layer_norm_epsilon)

    @classmethod
    def from_c(cls, c: _lib.pg_gpt2_config) -> "Gpt2Config":
        return cls(c.vocab_size, c.n_positions, c.n_embd, c.n_layer, c.n_head, c.n_inner,
                   c.layer_norm_epsilon)

    @classmethod
    def from_json_file(cls, path) -> "Gpt2Config":
        """load_config (src/models/gpt2/rust.rs:696-711): a Hugging Face config.json."""
        c = _lib.pg_gpt2_config()
        _check(_lib.load().pg_gpt2_load_config(str(path).encode(), C.byref(c)))
        return cls.from_c(c)


@dataclass
class Gpt2BlockWeights:
    """Gpt2BlockWeights (src/models/gpt2/rust.rs:111-125); matrices in HF [in,out] layout."""
    ln_1_g: np.ndarray
    ln_1_b: np.ndarray
    c_attn_w: np.ndarray
    c_attn_b: np.ndarray
    c_proj_w: np.ndarray
    c_proj_b: np.ndarray
    ln_2_g: np.ndarray
    ln_2_b: np.ndarray
    c_fc_w: np.ndarray
    c_fc_b: np.ndarray
    c_proj_mlp_w: np.ndarray
    c_proj_mlp_b: np.ndarray


@dataclass
class Gpt2Weights:
    """Gpt2Weights (src/models/gpt2/rust.rs:102-109): flat f32 arrays."""
    wte: np.ndarray
    wpe: np.ndarray
    blocks: List[Gpt2BlockWeights]
    ln_f_g: np.ndarray
    ln_f_b: np.ndarray


def _tensor(arr: np.ndarray, keep: list) -> _lib.pg_tensor:
    a = np.ascontiguousarray(arr, dtype=np.float32).reshape(-1)
    keep.append(a)
    return _lib.pg_tensor(_lib.f32p(a), a.size)


def weights_view(weights: Gpt2Weights, keep: list) -> _lib.pg_gpt2_weights_view:
    """Build the C view; `keep` receives the arrays that must outlive the call."""
    blocks = (_lib.pg_gpt2_block_view * max(len(weights.blocks), 1))()
    for i, b in enumerate(weights.blocks):
        for name in _lib.BLOCK_FIELDS:
            setattr(blocks[i], name, _tensor(getattr(b, name), keep))
    keep.append(blocks)
    return _lib.pg_gpt2_weights_view(_tensor(weights.wte, keep), _tensor(weights.wpe, keep),
                                     _tensor(weights.ln_f_g, keep), _tensor(weights.ln_f_b, keep),
                                     C.cast(blocks, C.POINTER(_lib.pg_gpt2_block_view)),
                                     len(weights.blocks))


def load_weights(path, cfg: Gpt2Config) -> Gpt2Weights:
    """load_weights (src/models/gpt2/rust.rs:713-771) into host arrays: Hugging Face tensor
    names, each tried bare and then with the `transformer.` prefix.  (Gpt2Model.from_dir
    does the same inside the library without host copies.)"""
    store = TensorStore(path)

    def tensor(name: str, shape) -> np.ndarray:
        found = store.optional_f32(name, shape)
        return found if found is not None else store.required_f32("transformer." + name, shape)

    c, i = cfg.n_embd, cfg.n_inner
    blocks = []
    for layer in range(cfg.n_layer):
        p = f"h.{layer}"
        blocks.append(Gpt2BlockWeights(
            ln_1_g=tensor(f"{p}.ln_1.weight", [c]), ln_1_b=tensor(f"{p}.ln_1.bias", [c]),
            c_attn_w=tensor(f"{p}.attn.c_attn.weight", [c, 3 * c]),
            c_attn_b=tensor(f"{p}.attn.c_attn.bias", [3 * c]),
            c_proj_w=tensor(f"{p}.attn.c_proj.weight", [c, c]),
            c_proj_b=tensor(f"{p}.attn.c_proj.bias", [c]),
            ln_2_g=tensor(f"{p}.ln_2.weight", [c]), ln_2_b=tensor(f"{p}.ln_2.bias", [c]),
            c_fc_w=tensor(f"{p}.mlp.c_fc.weight", [c, i]), c_fc_b=tensor(f"{p}.mlp.c_fc.bias", [i]),
            c_proj_mlp_w=tensor(f"{p}.mlp.c_proj.weight", [i, c]),
            c_proj_mlp_b=tensor(f"{p}.mlp.c_proj.bias", [c])))
    return Gpt2Weights(wte=tensor("wte.weight", [cfg.vocab_size, c]),
                       wpe=tensor("wpe.weight", [cfg.n_positions, c]), blocks=blocks,
                       ln_f_g=tensor("ln_f.weight", [c]), ln_f_b=tensor("ln_f.bias", [c]))


def Gpt2GenerationConfig(max_new_tokens: int) -> TextGenerationConfig:
    """Gpt2GenerationConfig::new (src/models/gpt2/options.rs:156-162): EOS 50256."""
    return TextGenerationConfig(max_new_tokens, eos_token_id=GPT2_EOS_TOKEN_ID)


class Gpt2KvCache(KvCache):
    """Gpt2KvCache (src/models/gpt2/rust.rs:177-249): K and V panels of n_positions rows."""

    def read_layer(self, layer: int, which: int, b: int = 0) -> np.ndarray:
        cfg = self._model.config
        out = np.empty((cfg.n_head, cfg.n_positions, cfg.head_dim()), dtype=np.float32)
        _check(_lib.load().pg_kv_cache_read_layer(self._h, b, layer, which, _lib.f32p(out),
                                                  out.size))
        return out


class Gpt2Model(Model):
    """Gpt2Model (src/models/gpt2/rust.rs:141-148, 798-1051) on the HIP backend;
    implements AutoregressiveDecoder (src/models/autoregressive.rs:9-31)."""

    CACHE = Gpt2KvCache

    def __init__(self, handle, config: Gpt2Config):
        super().__init__(handle)
        self.config = config

    @classmethod
    def new(cls, config: Gpt2Config, weights: Gpt2Weights,
            hip_config: Optional[Gpt2HipConfig] = None) -> "Gpt2Model":
        keep: list = []
        cfg = config.to_c()
        view = weights_view(weights, keep)
        opts = (hip_config or Gpt2HipConfig()).to_c()
        h = C.c_void_p()
        _check(_lib.load().pg_gpt2_create(C.byref(cfg), C.byref(view), C.byref(opts), C.byref(h)))
        return cls(h, config)

    @classmethod
    def from_dir(cls, model_dir, hip_config: Optional[Gpt2HipConfig] = None) -> "Gpt2Model":
        """Gpt2Runtime::from_dir_with_backend without the tokenizer
        (src/models/gpt2/rust.rs:382-393): `config.json` + `model.safetensors`."""
        opts = (hip_config or Gpt2HipConfig()).to_c()
        h = C.c_void_p()
        lib = _lib.load()
        _check(lib.pg_gpt2_create_from_dir(str(model_dir).encode(), C.byref(opts), C.byref(h)))
        cfg = _lib.pg_gpt2_config()
        _check(lib.pg_gpt2_get_config(h, C.byref(cfg)))
        return cls(h, Gpt2Config.from_c(cfg))
