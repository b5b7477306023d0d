"""What the models of every architecture share on the Python side: errors, options, statistics,
the cache and logits handles, the generation calls and the sampler, over the HIP C ABI.

Names, argument meaning and error behaviour follow the reference (src/models/gpt2/rust.rs,
src/models/autoregressive.rs, src/models/generation.rs).  All compute happens inside
libpuppygrad_hip.so.
"""
from __future__ import annotations

import ctypes as C
from dataclasses import dataclass
from typing import Callable, List, Optional, Sequence

import numpy as np

from . import _lib


class Gpt2Error(Exception):
    """Gpt2Error (src/models/gpt2/error.rs:4-21); `kind` is the variant name."""

    PREFIX = {
        "Asset": "GPT-2 asset error: ",
        "InvalidConfig": "invalid GPT-2 config: ",
        "InvalidInput": "invalid GPT-2 input: ",
        "InvalidWeights": "invalid GPT-2 weights: ",
        "Backend": "GPT-2 hip backend error: ",
    }

    def __init__(self, kind: str, msg: str):
        super().__init__(self.PREFIX[kind] + msg)
        self.kind = kind
        self.msg = msg


_KIND = {_lib.PG_ASSET: "Asset", _lib.PG_INVALID_CONFIG: "InvalidConfig",
         _lib.PG_INVALID_INPUT: "InvalidInput", _lib.PG_INVALID_WEIGHTS: "InvalidWeights",
         _lib.PG_BACKEND: "Backend"}


def _check(status: int) -> None:
    if status != _lib.PG_OK:
        msg = _lib.load().pg_last_error_message().decode()
        raise Gpt2Error(_KIND.get(status, "Backend"), msg)


class TensorStore:
    """TensorStore (src/models/safetensors.rs:93-138) over a mapped .safetensors file.
    Arrays returned are read-only views into the mapping and keep the store alive."""

    def __init__(self, path):
        h = C.c_void_p()
        _check(_lib.load().pg_tensor_store_open(str(path).encode(), C.byref(h)))
        self._h = h

    def __del__(self):
        h = getattr(self, "_h", None)
        if h:
            _lib.load().pg_tensor_store_close(h)
            self._h = None

    def __len__(self) -> int:
        return int(_lib.load().pg_tensor_store_len(self._h))

    def _view(self, t: _lib.pg_tensor, shape) -> np.ndarray:
        n = int(t.len)
        if n == 0:
            arr = np.zeros(0, np.float32)
        else:
            addr = C.cast(t.data, C.c_void_p).value
            arr = np.frombuffer((C.c_float * n).from_address(addr), np.float32)
        arr = arr.reshape(tuple(shape))
        arr.flags.writeable = False  # the mapping is read-only
        return _StoreArray.wrap(arr, self)

    def required_f32(self, name: str, expected_shape: Sequence[int]) -> np.ndarray:
        shape = (C.c_uint64 * max(len(expected_shape), 1))(*expected_shape)
        t = _lib.pg_tensor()
        _check(_lib.load().pg_tensor_store_required_f32(self._h, name.encode(), shape,
                                                        len(expected_shape), C.byref(t)))
        return self._view(t, expected_shape)

    def optional_f32(self, name: str, expected_shape: Sequence[int]) -> Optional[np.ndarray]:
        shape = (C.c_uint64 * max(len(expected_shape), 1))(*expected_shape)
        t = _lib.pg_tensor()
        found = C.c_int32(0)
        _check(_lib.load().pg_tensor_store_optional_f32(self._h, name.encode(), shape,
                                                        len(expected_shape), C.byref(found),
                                                        C.byref(t)))
        return self._view(t, expected_shape) if found.value else None


class _StoreArray(np.ndarray):
    """An ndarray that holds a reference to the TensorStore whose mapping it views."""

    @classmethod
    def wrap(cls, arr: np.ndarray, store: TensorStore) -> "np.ndarray":
        out = arr.view(cls)
        out._store = store
        return out

    def __array_finalize__(self, obj):
        self._store = getattr(obj, "_store", None)


@dataclass
class Gpt2HipConfig:
    """The per-backend knobs that sit where Gpt2RustConfig does
    (src/models/gpt2/options.rs:54-96)."""
    device: int = 0
    weight_storage: int = _lib.PG_STORE_F32
    decode_path: int = _lib.PG_DECODE_AUTO
    prefill_path: int = 0  # 0: GEMM prefill for prompts of seq_gemm_min_tokens and more, 1: token by token
    # tunables (0 = built-in default): what the autotune scan varies and puppygrad-tune.json holds
    attn_item_keys: int = 0
    attn_blocks_per_cu: int = 0
    gemm_split_items_per_cu: int = 0
    gemm_b9_min_rows: int = 0
    seq_gemm_min_tokens: int = 0

    def to_c(self) -> _lib.pg_hip_options:
        return _lib.pg_hip_options(self.device, self.weight_storage, self.decode_path,
                                   self.prefill_path, self.attn_item_keys, self.attn_blocks_per_cu,
                                   self.gemm_split_items_per_cu, self.gemm_b9_min_rows,
                                   self.seq_gemm_min_tokens, 0)


@dataclass
class TextGenerationConfig:
    """TextGenerationConfig (src/models/generation.rs:61-89)."""
    max_new_tokens: int
    eos_token_id: Optional[int] = None
    temperature: float = 0.0
    top_p: Optional[float] = None
    top_k: Optional[int] = None
    seed: int = 299_792_458
    repeat_penalty: float = 1.0
    repeat_last_n: int = 128

    def to_c(self) -> _lib.pg_sampling:
        return _lib.pg_sampling(self.temperature, int(self.top_p is not None),
                                self.top_p if self.top_p is not None else 0.0,
                                int(self.top_k is not None),
                                self.top_k if self.top_k is not None else 0,
                                self.repeat_penalty, self.repeat_last_n)

    def validate(self) -> None:
        s = self.to_c()
        _check(_lib.load().pg_sampling_validate(C.byref(s)))


@dataclass
class Gpt2OperationProfile:
    """Gpt2OperationProfile (src/models/gpt2/rust.rs:336-347), seconds per bucket.  LayerNorm
    runs inside the projection that consumes it on this backend: its bucket stays 0."""
    tokenization: float = 0.0
    layer_norm: float = 0.0
    qkv_projection: float = 0.0
    attention: float = 0.0
    attention_projection: float = 0.0
    mlp_fc_projection: float = 0.0
    mlp_projection: float = 0.0
    final_logits: float = 0.0
    decoding: float = 0.0


@dataclass
class GenerationStats:
    """GenerationStats (src/models/generation.rs:129-180)."""
    prompt_tokens: int = 0
    generated_tokens: int = 0
    prefill_time: float = 0.0
    decode_time: float = 0.0
    first_token_time: Optional[float] = None
    gpu_decode_time: float = 0.0
    tokenize_time: float = 0.0  # host time of the prompt's encode; set by Gpt2Runtime

    @property
    def total_generation_time(self) -> float:
        return self.prefill_time + self.decode_time

    def total_model_tokens(self) -> int:
        return self.prompt_tokens + self.generated_tokens

    @staticmethod
    def _rate(tokens: int, seconds: float) -> float:
        return 0.0 if seconds == 0.0 else tokens / seconds

    def prefill_tokens_per_second(self) -> float:
        return self._rate(self.prompt_tokens, self.prefill_time)

    def decode_tokens_per_second(self) -> float:
        return self._rate(self.generated_tokens, self.decode_time)

    def total_tokens_per_second(self) -> float:
        return self._rate(self.total_model_tokens(), self.total_generation_time)

    def average_decode_token_time(self) -> Optional[float]:
        if self.generated_tokens == 0:
            return None
        return self.decode_time / self.generated_tokens


def _u32(ids: Sequence[int]) -> np.ndarray:
    arr = np.asarray(ids, dtype=np.int64).reshape(-1)
    if arr.size and (arr.min() < 0 or arr.max() > 0xFFFFFFFF):
        raise Gpt2Error("InvalidInput", "token id out of u32 range")
    return arr.astype(np.uint32)


class DeviceLogits:
    """The `Logits` associated type of the HIP decoder: a device-resident buffer
    owned by its cache, valid until the next call that takes that cache."""

    def __init__(self, handle: int, cache: "KvCache"):
        self._h = handle
        self._cache = cache

    @property
    def rows(self) -> int:
        return _lib.load().pg_logits_rows(self._h)

    @property
    def vocab(self) -> int:
        return _lib.load().pg_logits_vocab(self._h)

    def to_host(self) -> np.ndarray:
        out = np.empty((self.rows, self.vocab), dtype=np.float32)
        _check(_lib.load().pg_logits_copy_to_host(self._h, _lib.f32p(out), out.size))
        return out[0] if self.rows == 1 else out

    def argmax(self) -> np.ndarray:
        out = np.empty(self.rows, dtype=np.uint32)
        _check(_lib.load().pg_logits_argmax(self._h, _lib.u32p(out)))
        return out


class KvCache:
    """The state of `batch` sequences that step together, in HBM: Gpt2KvCache
    (src/models/gpt2/rust.rs:177-249) for GPT-2, chunks of keys and values, recurrent matrices
    and convolution inputs for a stack model."""

    def __init__(self, model: "Model", batch: int = 1):
        h = C.c_void_p()
        _check(_lib.load().pg_kv_cache_create(model._h, batch, C.byref(h)))
        self._h = h
        self._model = model  # keeps the model alive

    def __del__(self):
        h = getattr(self, "_h", None)
        if h:
            _lib.load().pg_kv_cache_destroy(h)
            self._h = None

    @property
    def seq_len(self) -> int:
        return _lib.load().pg_kv_cache_seq_len(self._h)

    @seq_len.setter
    def seq_len(self, n: int) -> None:
        _check(_lib.load().pg_kv_cache_set_seq_len(self._h, n))

    @property
    def max_seq_len(self) -> int:
        return _lib.load().pg_kv_cache_max_seq_len(self._h)

    @property
    def batch(self) -> int:
        return _lib.load().pg_kv_cache_batch(self._h)

    def clear(self) -> None:
        _check(_lib.load().pg_kv_cache_clear(self._h))


class Model:
    """A model on the HIP backend, whatever its architecture; implements AutoregressiveDecoder
    (src/models/autoregressive.rs:9-31) and the generation calls of the reference's Gpt2Model
    (src/models/gpt2/rust.rs:798-1051).  `models.load_model` makes one from a directory."""

    CACHE = KvCache

    def __init__(self, handle):
        self._h = handle

    def __del__(self):
        h = getattr(self, "_h", None)
        if h:
            _lib.load().pg_model_destroy(h)
            self._h = None

    @property
    def architecture(self) -> str:
        return _lib.load().pg_model_architecture(self._h).decode()

    def _info(self) -> _lib.pg_model_info:
        info = _lib.pg_model_info()
        _check(_lib.load().pg_model_get_info(self._h, C.byref(info)))
        return info

    @property
    def vocab_size(self) -> int:
        return self._info().vocab_size

    def describe(self) -> str:
        buf = C.create_string_buffer(256)
        _check(_lib.load().pg_model_describe(self._h, buf, len(buf)))
        return buf.value.decode()

    # -- AutoregressiveDecoder -------------------------------------------------
    def max_context_len(self) -> int:
        return self._info().max_positions

    def new_kv_cache(self, batch: int = 1) -> KvCache:
        return self.CACHE(self, batch)

    def new_cache(self) -> KvCache:
        return self.new_kv_cache()

    def prefill(self, input_ids: Sequence[int], cache: KvCache) -> DeviceLogits:
        ids = _u32(input_ids)
        out = C.c_void_p()
        _check(_lib.load().pg_model_prefill(self._h, cache._h, _lib.u32p(ids), ids.size,
                                           C.byref(out)))
        return DeviceLogits(out, cache)

    def prefill_profiled(self, input_ids: Sequence[int], cache: KvCache):
        """prefill_profiled (rust.rs:906-927): the logits and the per-operation times."""
        ids = _u32(input_ids)
        out = C.c_void_p()
        prof = _lib.pg_gpt2_operation_profile()
        _check(_lib.load().pg_model_prefill_profiled(self._h, cache._h, _lib.u32p(ids), ids.size,
                                                    C.byref(out), C.byref(prof)))
        return DeviceLogits(out, cache), Gpt2OperationProfile(
            **{f[0][:-2]: getattr(prof, f[0]) for f in prof._fields_})

    def extend(self, input_ids: Sequence[int], cache: KvCache,
               want: Optional[Sequence[int]] = None) -> Optional[DeviceLogits]:
        """The next tokens of the cache's sequence in one portion, from the state earlier calls
        left.  `want` (the last token by default) are the increasing places among them whose
        logits are returned, one row each; None when it is empty."""
        ids = _u32(input_ids)
        places = [ids.size - 1] if want is None else [int(w) for w in want]
        if any(w < 0 for w in places):
            raise Gpt2Error("InvalidInput", "wanted places must increase and lie inside the portion")
        arr = (C.c_size_t * max(len(places), 1))(*places)
        out = C.c_void_p()
        _check(_lib.load().pg_model_extend(self._h, cache._h, _lib.u32p(ids), ids.size, arr,
                                           len(places), C.byref(out)))
        return DeviceLogits(out, cache) if places else None

    def forward_one(self, token_id: int, cache: KvCache) -> DeviceLogits:
        if token_id < 0 or token_id > 0xFFFFFFFF:
            raise Gpt2Error("InvalidInput", f"token id {token_id} exceeds vocab_size "
                                            f"{self.vocab_size}")
        out = C.c_void_p()
        _check(_lib.load().pg_model_forward_one(self._h, cache._h, token_id, C.byref(out)))
        return DeviceLogits(out, cache)

    def select_next_token(self, logits: DeviceLogits) -> int:
        return int(logits.argmax()[0])

    # -- batched forms ---------------------------------------------------------
    def prefill_batch(self, input_ids: np.ndarray, cache: KvCache) -> DeviceLogits:
        ids = np.ascontiguousarray(np.asarray(input_ids, dtype=np.uint32))
        if ids.ndim != 2 or ids.shape[0] != cache.batch:
            raise Gpt2Error("InvalidInput", "prefill_batch expects ids of shape [batch][n]")
        out = C.c_void_p()
        _check(_lib.load().pg_model_prefill_batch(self._h, cache._h, _lib.u32p(ids), ids.shape[1],
                                                 C.byref(out)))
        return DeviceLogits(out, cache)

    def forward_one_batch(self, token_ids: Sequence[int], cache: KvCache) -> DeviceLogits:
        ids = _u32(token_ids)
        if ids.size != cache.batch:
            raise Gpt2Error("InvalidInput", "forward_one_batch expects one id per sequence")
        out = C.c_void_p()
        _check(_lib.load().pg_model_forward_one_batch(self._h, cache._h, _lib.u32p(ids),
                                                     C.byref(out)))
        return DeviceLogits(out, cache)

    # -- full-sequence forward (rust.rs:831-882) ---------------------------------
    def forward(self, input_ids: Sequence[int]) -> "Gpt2Output":
        ids = _u32(input_ids)
        out = np.empty((max(ids.size, 1), self.vocab_size), dtype=np.float32)
        _check(_lib.load().pg_model_forward(self._h, _lib.u32p(ids), ids.size, _lib.f32p(out),
                                           ids.size * self.vocab_size))
        return Gpt2Output(out[:ids.size], ids.size, self.vocab_size)

    # -- generation (rust.rs:884-900, 1008-1027) ---------------------------------
    def generate_greedy(self, input_ids: Sequence[int], max_new_tokens: int) -> List[int]:
        """generate_greedy: a full forward per new token (rust.rs:884-900)."""
        tokens = [int(t) for t in input_ids]
        _check_nonempty(tokens)
        for _ in range(max_new_tokens):
            if len(tokens) >= self.max_context_len():
                break
            out = self.forward(tokens)
            tokens.append(argmax_logits(out.last_logits()))
        return tokens

    def generate_greedy_cached(self, input_ids: Sequence[int], max_new_tokens: int) -> List[int]:
        return self.stream_greedy_tokens(input_ids, max_new_tokens, lambda _t: None)

    def stream_greedy_tokens(self, input_ids: Sequence[int], max_new_tokens: int,
                             on_token: Callable[[int], None]) -> List[int]:
        return generate(self, input_ids, max_new_tokens, on_token)

    def decode_greedy(self, cache: KvCache, max_new: int,
                      eos: Optional[int] = None) -> "tuple[List[int], GenerationStats]":
        """The greedy loop with the token kept on the device (pg_model_decode_greedy)."""
        out = np.empty(max(max_new, 1), dtype=np.uint32)
        n = C.c_uint32()
        st = _lib.pg_generation_stats()
        _check(_lib.load().pg_model_decode_greedy(self._h, cache._h, max_new,
                                                 -1 if eos is None else eos, _lib.u32p(out),
                                                 C.byref(n), C.byref(st)))
        return [int(t) for t in out[:n.value]], _stats(st)

    def decode_greedy_batch(self, cache: KvCache,
                            steps: int) -> "tuple[np.ndarray, GenerationStats]":
        out = np.empty((max(steps, 1), cache.batch), dtype=np.uint32)
        st = _lib.pg_generation_stats()
        _check(_lib.load().pg_model_decode_greedy_batch(self._h, cache._h, steps, _lib.u32p(out),
                                                       C.byref(st)))
        return out[:st.generated_tokens], _stats(st)

    def stream_token_ids_with_stats(self, input_ids: Sequence[int],
                                    generation: TextGenerationConfig,
                                    on_token: Optional[Callable[[int], None]] = None,
                                    profiled: bool = False):
        """Gpt2Runtime::stream_token_ids_with_stats with ids in place of a prompt
        string (rust.rs:548-634).  With profiled=True every forward runs as one launch per
        operation, timed into a Gpt2OperationProfile, and a third value is returned."""
        ids = _u32(input_ids)
        out = np.empty(ids.size + generation.max_new_tokens + 1, dtype=np.uint32)
        n = C.c_size_t()
        st = _lib.pg_generation_stats()
        samp = generation.to_c()
        err: list = []

        def _cb(tok, _user):
            try:
                if on_token is not None:
                    on_token(int(tok))
                return 0
            except Exception as e:  # surfaced after the C call returns
                err.append(e)
                return 1

        cb = _lib.ON_TOKEN(_cb)
        args = (self._h, _lib.u32p(ids), ids.size, generation.max_new_tokens,
                -1 if generation.eos_token_id is None else generation.eos_token_id, C.byref(samp),
                generation.seed, cb, None, _lib.u32p(out), C.byref(n), C.byref(st))
        prof = _lib.pg_gpt2_operation_profile()
        if profiled:
            status = _lib.load().pg_model_stream_token_ids_profiled(*args, C.byref(prof))
        else:
            status = _lib.load().pg_model_stream_token_ids_with_stats(*args)
        if err:
            raise err[0]
        _check(status)
        tokens = [int(t) for t in out[:n.value]]
        if profiled:
            return tokens, _stats(st), Gpt2OperationProfile(
                **{f[0][:-2]: getattr(prof, f[0]) for f in prof._fields_})
        return tokens, _stats(st)


def _stats(st: _lib.pg_generation_stats) -> GenerationStats:
    return GenerationStats(st.prompt_tokens, st.generated_tokens, st.prefill_s, st.decode_s,
                           st.first_token_s if st.first_token_s >= 0 and st.generated_tokens else None,
                           st.gpu_decode_s)


def _check_nonempty(tokens) -> None:
    if len(tokens) == 0:
        raise Gpt2Error("InvalidInput", "input_ids must not be empty")


@dataclass
class Gpt2Output:
    """Gpt2Output (src/models/gpt2/rust.rs:150-175)."""
    logits: np.ndarray
    seq_len: int
    vocab_size: int

    def logits_for_position(self, pos: int) -> np.ndarray:
        if pos >= self.seq_len:
            raise Gpt2Error("InvalidInput",
                            f"position {pos} out of range for seq_len {self.seq_len}")
        return self.logits[pos]

    def last_logits(self) -> np.ndarray:
        if self.seq_len == 0:
            raise Gpt2Error("InvalidInput", "empty sequence")
        return self.logits_for_position(self.seq_len - 1)


def argmax_logits(values: np.ndarray) -> int:
    """argmax_logits (src/models/generation.rs:269-279) on a host vector, computed
    on the device through pg_op_argmax."""
    v = np.ascontiguousarray(values, dtype=np.float32).reshape(-1)
    out = C.c_uint32()
    _check(_lib.load().pg_op_argmax(0, _lib.f32p(v), v.size, C.byref(out)))
    return int(out.value)


def generate(model, input_ids: Sequence[int], max_new_tokens: int,
             on_token: Callable[[int], None]) -> List[int]:
    """autoregressive::generate (src/models/autoregressive.rs:61-87)."""
    cache = model.new_cache()
    logits = model.prefill(input_ids, cache)
    tokens = [int(t) for t in input_ids]
    for _ in range(max_new_tokens):
        if len(tokens) >= model.max_context_len():
            break
        nxt = model.select_next_token(logits)
        tokens.append(nxt)
        on_token(nxt)
        logits = model.forward_one(nxt, cache)
    return tokens


class LogitsSampler:
    """LogitsSampler (src/models/generation.rs:209-241) over device logits."""

    def __init__(self, seed: int):
        self._rng = _lib.pg_rng_state()
        _lib.load().pg_rng_seed(C.byref(self._rng), seed)

    def select_next_token(self, logits: DeviceLogits, history: Sequence[int],
                          config: TextGenerationConfig, row: int = 0) -> int:
        hist = _u32(history)
        samp = config.to_c()
        out = C.c_uint32()
        _check(_lib.load().pg_logits_sample(logits._h, row, _lib.u32p(hist), hist.size,
                                            C.byref(samp), C.byref(self._rng), C.byref(out)))
        return int(out.value)
