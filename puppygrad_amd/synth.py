"""Seeded synthetic GPT-2 weights and token ids, shared by tests and bench.

Weights are N(0, std) from the reference's splitmix64 (src/models/generation.rs:244-267)
through Box-Muller, generated inside libpuppygrad_hip.so (pg_synth_normal_f32).
One stream per seed; tensors take consecutive ranges of it in this order:
wte, wpe, then per layer c_attn_w, c_proj_w, c_fc_w, c_proj_mlp_w, all in the HF
[in,out] layout.  LayerNorm gamma = 1, beta = 0 and linear biases = 0 unless
`perturb` is set, in which case they get small seeded values so that tests cover
those terms.
"""
from __future__ import annotations

import numpy as np

from . import _lib
from .gpt2 import Gpt2BlockWeights, Gpt2Config, Gpt2Weights

GPT2_SMALL = dict(vocab_size=50257, n_positions=1024, n_embd=768, n_layer=12, n_head=12)
GPT2_MEDIUM = dict(vocab_size=50257, n_positions=1024, n_embd=1024, n_layer=24, n_head=16)
GPT2_LARGE = dict(vocab_size=50257, n_positions=1024, n_embd=1280, n_layer=36, n_head=20)
GPT2_XL = dict(vocab_size=50257, n_positions=1024, n_embd=1600, n_layer=48, n_head=25)

WEIGHT_SEED_BASE = 0x5EED_0000
TOKEN_SEED_BASE = 0x70C0_0000


def normal_f32(n: int, seed: int, first: int, std: float = 0.02) -> np.ndarray:
    out = np.empty(n, dtype=np.float32)
    _lib.load().pg_synth_normal_f32(_lib.f32p(out), n, seed, first, std)
    return out


def token_ids(n: int, seed: int, vocab: int) -> np.ndarray:
    out = np.empty(n, dtype=np.uint32)
    _lib.load().pg_synth_token_ids(_lib.u32p(out), n, seed, vocab)
    return out


def random_weights(cfg: Gpt2Config, seed: int, std: float = 0.02,
                   perturb: bool = False) -> Gpt2Weights:
    C, I = cfg.n_embd, cfg.n_inner
    pos = 0

    def take(n):
        nonlocal pos
        a = normal_f32(n, seed, pos, std)
        pos += n
        return a

    wte = take(cfg.vocab_size * C)
    wpe = take(cfg.n_positions * C)
    blocks = []
    for _ in range(cfg.n_layer):
        c_attn_w = take(C * 3 * C)
        c_proj_w = take(C * C)
        c_fc_w = take(C * I)
        c_proj_mlp_w = take(I * C)
        blocks.append(Gpt2BlockWeights(
            ln_1_g=np.ones(C, np.float32), ln_1_b=np.zeros(C, np.float32),
            c_attn_w=c_attn_w, c_attn_b=np.zeros(3 * C, np.float32),
            c_proj_w=c_proj_w, c_proj_b=np.zeros(C, np.float32),
            ln_2_g=np.ones(C, np.float32), ln_2_b=np.zeros(C, np.float32),
            c_fc_w=c_fc_w, c_fc_b=np.zeros(I, np.float32),
            c_proj_mlp_w=c_proj_mlp_w, c_proj_mlp_b=np.zeros(C, np.float32)))
    w = Gpt2Weights(wte, wpe, blocks, np.ones(C, np.float32), np.zeros(C, np.float32))
    if perturb:
        # A second stream (seed + 1) for the terms the default init leaves at 0 / 1.
        p = 0

        def small(n, centre):
            nonlocal p
            a = normal_f32(n, seed + 1, p, 0.1) + np.float32(centre)
            p += n
            return a.astype(np.float32)

        for b in w.blocks:
            b.ln_1_g, b.ln_1_b = small(C, 1.0), small(C, 0.0)
            b.c_attn_b, b.c_proj_b = small(3 * C, 0.0), small(C, 0.0)
            b.ln_2_g, b.ln_2_b = small(C, 1.0), small(C, 0.0)
            b.c_fc_b, b.c_proj_mlp_b = small(I, 0.0), small(C, 0.0)
        w.ln_f_g, w.ln_f_b = small(C, 1.0), small(C, 0.0)
    return w


def patterned(n: int, scale: float) -> np.ndarray:
    """The reference's test pattern (src/models/gpt2/rust.rs:2117-2121)."""
    i = np.arange(n, dtype=np.int64)
    return (((i * 17 + 11) % 23).astype(np.float32) - np.float32(11.0)) * np.float32(scale)


def tiny_config() -> Gpt2Config:
    """tiny_config (src/models/gpt2/rust.rs:2082-2092)."""
    return Gpt2Config(vocab_size=8, n_positions=5, n_embd=4, n_layer=1, n_head=2, n_inner=8,
                      layer_norm_epsilon=1e-5)


def tiny_weights(cfg: Gpt2Config) -> Gpt2Weights:
    """tiny_weights (src/models/gpt2/rust.rs:2094-2115)."""
    C, I = cfg.n_embd, cfg.n_inner
    one, zero = (lambda n: np.ones(n, np.float32)), (lambda n: np.zeros(n, np.float32))
    return Gpt2Weights(
        wte=patterned(cfg.vocab_size * C, 0.03), wpe=patterned(cfg.n_positions * C, 0.02),
        blocks=[Gpt2BlockWeights(
            ln_1_g=one(C), ln_1_b=zero(C), c_attn_w=patterned(C * 3 * C, 0.01),
            c_attn_b=zero(3 * C), c_proj_w=patterned(C * C, 0.015), c_proj_b=zero(C),
            ln_2_g=one(C), ln_2_b=zero(C), c_fc_w=patterned(C * I, 0.01), c_fc_b=zero(I),
            c_proj_mlp_w=patterned(I * C, 0.012), c_proj_mlp_b=zero(C))],
        ln_f_g=one(C), ln_f_b=zero(C))


def round_bf16(a: np.ndarray) -> np.ndarray:
    """f32 -> bf16 (round to nearest even) -> f32, as the bf16 weight storage does."""
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32)
    r = (u + np.uint32(0x7FFF) + ((u >> np.uint32(16)) & np.uint32(1))) & np.uint32(0xFFFF0000)
    return r.view(np.float32)


def bf16_rounded(w: Gpt2Weights) -> Gpt2Weights:
    """The weights a bf16-storage model really multiplies with: wte and the four block
    matrices rounded to bf16; LayerNorm parameters, biases and wpe untouched."""
    blocks = [Gpt2BlockWeights(
        ln_1_g=b.ln_1_g, ln_1_b=b.ln_1_b, c_attn_w=round_bf16(b.c_attn_w), c_attn_b=b.c_attn_b,
        c_proj_w=round_bf16(b.c_proj_w), c_proj_b=b.c_proj_b, ln_2_g=b.ln_2_g, ln_2_b=b.ln_2_b,
        c_fc_w=round_bf16(b.c_fc_w), c_fc_b=b.c_fc_b, c_proj_mlp_w=round_bf16(b.c_proj_mlp_w),
        c_proj_mlp_b=b.c_proj_mlp_b) for b in w.blocks]
    return Gpt2Weights(wte=round_bf16(w.wte), wpe=w.wpe, blocks=blocks, ln_f_g=w.ln_f_g,
                       ln_f_b=w.ln_f_b)


# ---- stack models (Tarepel, Movudra) --------------------------------------------------------------------
# Layers of a real model's proportions, by width: every layer has about the 12 width^2
# parameters of a GPT-2 layer of that width.  attn: heads of 64, key/value heads, chunk; delta
# and gla: heads with 128-value states; ff of either kind of layer.
STACK_SIZES = {
    768: dict(heads=12, kv_heads=4, chunk=512, delta=(8, 4, 128, 128), gla=(8, 64, 128), ff=(1088, 1696)),
    1280: dict(heads=20, kv_heads=5, chunk=512, delta=(12, 6, 128, 128), gla=(12, 64, 128), ff=(2048, 3072)),
    1600: dict(heads=25, kv_heads=5, chunk=512, delta=(16, 8, 128, 128), gla=(16, 64, 128), ff=(2560, 3712)),
}
STACK_GLA_RANK = 16


def tarepel_config(width: int, n_layer: int, vocab: int = 50257) -> dict:
    """A Tarepel config.json of STACK_SIZES[width]; every third layer is a gla layer."""
    z = STACK_SIZES[width]
    dh, dk, dd, dv = z["delta"]
    gh, gd, gv = z["gla"]
    parallel = {"type": "parallel", "mlp": {"kind": "dense", "ff": z["ff"][0]}, "mixer": {
        "left": {"heads": z["heads"], "kv_heads": z["kv_heads"], "dim": 64, "vdim": 64, "scale": 0.125,
                 "mask": {"size": z["chunk"]}, "rot": {"dims": 64, "base": 10000.0}},
        "right": {"heads": dh, "kv_heads": dk, "dim": dd, "vdim": dv, "conv": 4},
        "left_scale": 0.5, "right_scale": 1.0}}
    gla = {"type": "gla", "mlp": {"kind": "dense", "ff": z["ff"][1]},
           "mixer": {"heads": gh, "dim": gd, "vdim": gv, "tau": 8.0}}
    return {"architecture": "Tarepel", "vocab": vocab, "width": width, "norm": {"eps": 1e-6},
            "logit_scale": 1.0, "layers": [gla if i % 3 == 2 else parallel for i in range(n_layer)]}


# Movudra: mamba2 (heads, groups, state, vdim), channel_delta (heads, kv_heads, dim, vdim, rank of decay
# and gate), latent_attention (heads, dim, rot_dim, vdim, q_rank, kv_rank, window).
MOVUDRA_SIZES = {
    768: dict(mamba=(24, 1, 128, 64), delta=(6, 6, 128, 128, 128), latent=(8, 64, 32, 64, 384, 256, 512)),
    1280: dict(mamba=(40, 2, 128, 64), delta=(10, 10, 128, 128, 128), latent=(10, 128, 64, 128, 512, 512, 512)),
    1600: dict(mamba=(50, 2, 128, 64), delta=(16, 16, 128, 128, 128), latent=(16, 128, 64, 128, 768, 512, 512)),
}
MOVUDRA_EXPERTS, MOVUDRA_TOP = 8, 2


def movudra_config(width: int, n_layer: int, vocab: int = 50257) -> dict:
    """A Movudra config.json of MOVUDRA_SIZES[width]: the three mixers in turn, the first layer dense,
    the others with experts; a token meets about 12 width^2 parameters in every layer."""
    z = MOVUDRA_SIZES[width]
    H, G, N, e = z["mamba"]
    mamba = {"heads": H, "groups": G, "state": N, "vdim": e, "conv": 4, "norm_groups": G}
    n_mamba = width * (2 * H * e + 2 * G * N + H) + width * H * e
    H, G, d, e, r = z["delta"]
    delta = {"heads": H, "kv_heads": G, "dim": d, "vdim": e, "conv": 4}
    n_delta = width * (2 * G * d + 2 * H * e + H) + r * (2 * width + H * (d + e))
    H, d, rot, e, q, kv, window = z["latent"]
    latent = {"heads": H, "dim": d, "rot_dim": rot, "vdim": e, "q_rank": q, "kv_rank": kv, "scale": (d + rot) ** -0.5,
              "mask": {"size": window}, "rot": {"dims": rot, "base": 10000.0, "scaling": {
                  "factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
    n_latent = width * (q + kv + rot + H * e) + q * H * (d + rot) + kv * H * (d + e)
    layers = []
    for i in range(n_layer):
        kind, mixer, n = (("mamba2", mamba, n_mamba), ("channel_delta", delta, n_delta),
                          ("latent_attention", latent, n_latent))[i % 3]
        rest = 12 * width * width - n
        if i == 0:
            mlp = {"kind": "dense", "ff": round(rest / (2 * width * 32)) * 32}
        else:
            mlp = {"kind": "moe", "router": {"experts": MOVUDRA_EXPERTS, "top": MOVUDRA_TOP},
                   "expert": {"ff": round(rest / (3 * width * MOVUDRA_TOP * 32)) * 32}}
        layers.append({"type": kind, "mixer": mixer, "mlp": mlp})
    return {"architecture": "Movudra", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "layers": layers}


def movudra_tensor_shapes(cfg: dict, ranks=(128, 128)) -> "dict[str, tuple]":
    """Names and shapes of a Movudra model's tensors; ranks: of the decay and of the output gate."""
    C, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, C)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        q = p + "mix."
        out[p + "norm1"] = (C,)
        if layer["type"] == "mamba2":
            H, inner, gn = m["heads"], m["heads"] * m["vdim"], m["groups"] * m["state"]
            ch = inner + 2 * gn
            out.update({q + "in": (inner + ch + H, C), q + "conv": (ch, m["conv"]), q + "conv.b": (ch,), q + "dt_bias": (H,),
                        q + "A_log": (H,), q + "D": (H,), q + "norm": (inner,), q + "o": (C, inner)})
        elif layer["type"] == "channel_delta":
            H, qk, vv, hd = m["heads"], m["kv_heads"] * m["dim"], m["heads"] * m["vdim"], m["heads"] * m["dim"]
            for x, n in (("q", qk), ("k", qk), ("v", vv)):
                out.update({q + x: (n, C), q + x + ".conv": (n, m["conv"])})
            out.update({q + "b": (H, C), q + "A_log": (H,), q + "norm": (m["vdim"],), q + "a1": (ranks[0], C),
                        q + "a2": (hd, ranks[0]), q + "dt_bias": (hd,), q + "g1": (ranks[1], C), q + "g2": (vv, ranks[1]),
                        q + "o": (C, vv)})
        else:
            H, K = m["heads"], m["kv_rank"]
            out.update({q + "dq": (m["q_rank"], C), q + "dq.norm": (m["q_rank"],),
                        q + "uq": (H * (m["dim"] + m["rot_dim"]), m["q_rank"]), q + "dkv": (K + m["rot_dim"], C),
                        q + "dkv.norm": (K,), q + "uk": (H * m["dim"], K), q + "uv": (H * m["vdim"], K), q + "sink": (H,),
                        q + "o": (C, H * m["vdim"])})
        f = layer.get("mlp")
        if f:
            out[p + "norm2"] = (C,)
            q = p + "mlp."
            if f["kind"] == "dense":
                out.update({q + "up": (f["ff"], C), q + "up.b": (f["ff"],), q + "down": (C, f["ff"]), q + "down.b": (C,)})
            else:
                ff = f["expert"]["ff"]
                for e in range(f["router"]["experts"]):
                    out.update({f"{q}e{e}.gate": (ff, C), f"{q}e{e}.up": (ff, C), f"{q}e{e}.down": (C, ff)})
                out[q + "router"] = (f["router"]["experts"], C)
    out.update({"final.norm": (C,), "head": (V, C)})
    return out


def stack_tensor_shapes(cfg: dict, rank=None) -> "dict[str, tuple]":
    """Names and shapes of a stack model's tensors (rank: what config.json leaves to the tensors)."""
    if cfg["architecture"] == "Movudra":
        return movudra_tensor_shapes(cfg, *([] if rank is None else [rank]))
    return tarepel_tensor_shapes(cfg, *([] if rank is None else [rank]))


def tarepel_tensor_shapes(cfg: dict, rank: int = STACK_GLA_RANK) -> "dict[str, tuple]":
    """Names and shapes of a Tarepel model's tensors."""
    C, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, C)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out[p + "norm1"] = ()
        if layer["type"] == "parallel":
            L, R = m["left"], m["right"]
            hd, gd = L["heads"] * L["dim"], L["kv_heads"] * L["dim"]
            q = p + "mix.left."
            out.update({q + "q": (hd, C), q + "k": (gd, C), q + "pb": (L["heads"],), q + "o": (C, hd)})
            qk, vv, H = R["kv_heads"] * R["dim"], R["heads"] * R["vdim"], R["heads"]
            q = p + "mix.right."
            out.update({q + "q": (qk, C), q + "q.conv": (qk, R["conv"]), q + "k": (qk, C),
                        q + "k.conv": (qk, R["conv"]), q + "v": (vv, C), q + "v.conv": (vv, R["conv"]),
                        q + "b": (H, C), q + "A_log": (H,), q + "norm": (R["vdim"],), q + "a": (H, C),
                        q + "dt_bias": (H,), q + "g": (vv, C), q + "o": (C, vv)})
        else:
            qk, vv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            q = p + "mix."
            out.update({q + "q": (qk, C), q + "k": (qk, C), q + "v": (vv, C), q + "g": (vv, C),
                        q + "o": (C, vv), q + "norm": (m["vdim"],), q + "a1": (rank, C),
                        q + "a2": (qk, rank), q + "a2.b": (qk,)})
        out[p + "ls1"] = (C,)
        if layer.get("mlp"):
            ff = layer["mlp"]["ff"]
            out.update({p + "mlp.gate": (ff, C), p + "mlp.up": (ff, C), p + "mlp.down": (C, ff),
                        p + "ls2": (C,)})
    out.update({"final.norm": (), "head": (V, C)})
    return out


def bf16_bits(a: np.ndarray) -> np.ndarray:
    """The bf16 bit patterns (uint16) of f32 values, nearest even."""
    a = np.ascontiguousarray(a, np.float32)
    out = np.empty(a.shape, np.uint16)
    flat, dst, step = a.reshape(-1), out.reshape(-1), 1 << 18  # (a piece that stays in the CPU's cache)
    for i in range(0, flat.size, step):
        dst[i:i + step] = round_bf16(flat[i:i + step]).view(np.uint32) >> np.uint32(16)
    return out


def write_model_dir(path, cfg: dict, tensors) -> None:
    """config.json and a bf16 model.safetensors from an iterable of (name, f32 array)
    (arrays are taken one at a time)."""
    import json
    import os
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w", encoding="utf-8") as f:
        json.dump(cfg, f)
    header, at, body = {}, 0, os.path.join(path, "model.safetensors.body")
    with open(body, "wb") as f:
        for name, a in tensors:
            bits = bf16_bits(np.asarray(a, np.float32).reshape(-1))
            header[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [at, at + bits.nbytes]}
            at += bits.nbytes
            f.write(bits.tobytes())
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as f, open(body, "rb") as b:
        f.write(len(text).to_bytes(8, "little") + text)
        while True:
            part = b.read(1 << 24)
            if not part:
                break
            f.write(part)
    os.remove(body)


def stack_weights(cfg: dict, seed: int, std: float = 0.02):
    """(name, array) of seeded random weights: N(0, std), with norm gains of 1, layer scales of
    0.3, convolution taps around a mean filter and decays between a few and a few hundred
    tokens."""
    pos = 0
    for name, shape in stack_tensor_shapes(cfg).items():
        n = int(np.prod(shape, dtype=np.int64))
        a = normal_f32(n, seed, pos, std)
        pos += n
        last = name.split(".")[-1]
        if last.startswith("norm"):
            a = a + np.float32(1.0)
        elif last in ("ls1", "ls2"):
            a = a + np.float32(0.3)
        elif last == "conv":
            a = a * np.float32(10.0) + np.float32(1.0 / shape[1])
        elif last == "A_log":
            a = a * np.float32(20.0)
        elif last == "dt_bias":
            a = a * np.float32(40.0) - np.float32(3.0)
        elif name.endswith("a2.b"):
            a = a * np.float32(40.0) + np.float32(2.0)
        elif last == "D":
            a = a + np.float32(1.0)
        yield name, a.reshape(shape)
