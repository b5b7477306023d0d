"""The model registry: from a directory (config.json, model.safetensors) to the model class of its
architecture."""
from __future__ import annotations

import ctypes as C
import json
import os
from typing import Callable, Dict, Optional

from . import _lib
from .gpt2 import Gpt2Config, Gpt2Model
from .model import Gpt2HipConfig, Model, _check


class StackModel(Model):
    """A model whose config.json lists its layers with their mixers (Tarepel, Movudra).  `config` is that
    file's object.  Weights are stored as `hip_config.weight_storage` says (f32 or bf16); a cache
    has a fixed size and takes sequences of any length."""

    def __init__(self, handle, config: dict):
        super().__init__(handle)
        self.config = config

    @classmethod
    def from_handle(cls, handle, model_dir) -> "StackModel":
        with open(os.path.join(os.fspath(model_dir), "config.json"), encoding="utf-8") as f:
            return cls(handle, json.load(f))


def _gpt2(handle, model_dir) -> Gpt2Model:
    cfg = _lib.pg_gpt2_config()
    _check(_lib.load().pg_gpt2_get_config(handle, C.byref(cfg)))
    return Gpt2Model(handle, Gpt2Config.from_c(cfg))


# architecture (pg_model_architecture) -> what wraps its handle
ARCHITECTURES: Dict[str, Callable[..., Model]] = {"gpt2": _gpt2, "Tarepel": StackModel.from_handle,
                                           "Movudra": StackModel.from_handle}


def load_model(model_dir, hip_config: Optional[Gpt2HipConfig] = None) -> Model:
    """The model of a directory; config.json says which architecture it is."""
    opts = (hip_config or Gpt2HipConfig()).to_c()
    h = C.c_void_p()
    lib = _lib.load()
    _check(lib.pg_model_create_from_dir(os.fspath(model_dir).encode(), C.byref(opts), C.byref(h)))
    wrap = ARCHITECTURES[lib.pg_model_architecture(h).decode()]
    return wrap(h, model_dir)
