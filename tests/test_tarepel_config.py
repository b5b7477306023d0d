"""CPU-only: the Tarepel oracle's mechanisms in other forms than its own loops, and the errors of
the registry and of the config reader before any device work."""
import copy
import json

import numpy as np
import pytest

import oracle.tarepel as orc
from puppygrad_amd import Gpt2Error, load_model, synth

CFG = {"architecture": "Tarepel", "vocab": 19, "width": 20, "norm": {"eps": 1e-5}, "logit_scale": 0.5, "layers": [
    {"type": "parallel", "mlp": {"kind": "dense", "ff": 12}, "mixer": {
        "left": {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 6, "scale": 0.3, "mask": {"size": 5}, "rot": {"dims": 4, "base": 100.0}},
        "right": {"heads": 2, "kv_heads": 1, "dim": 4, "vdim": 6, "conv": 3}, "left_scale": 0.9, "right_scale": 1.4}},
    {"type": "gla", "mlp": None, "mixer": {"heads": 2, "dim": 4, "vdim": 6, "tau": 2.0}}]}


def test_rotation_depends_on_the_distance_only():
    g = np.random.default_rng(0)
    q, k = g.standard_normal(10), g.standard_normal(10)
    for dims in (10, 6, 0):
        dots = [orc.rotate(q, p + 7, dims, 30.0) @ orc.rotate(k, p, dims, 30.0) for p in (0, 3, 1000)]
        np.testing.assert_allclose(dots, dots[0], rtol=1e-9)
        np.testing.assert_array_equal(orc.rotate(q, 5, dims, 30.0)[dims:], q[dims:])
    # the complex form: value i + j value (i + dims / 2) times exp(j p f_i)
    z = (q[:5] + 1j * q[5:]) * np.exp(1j * 3 * 30.0 ** (-2 * np.arange(5) / 10))
    np.testing.assert_allclose(orc.rotate(q, 3, 10, 30.0), np.concatenate([z.real, z.imag]), rtol=1e-12)


def test_delta_rule_writes_a_value_that_is_read_back():
    g = np.random.default_rng(1)
    k, v = orc.unit(g.standard_normal(6)), g.standard_normal(4)
    S = g.standard_normal((6, 4))
    S2, o = orc.delta_step(S, k, k, v, 1.0, 1.0)  # beta 1, no decay: reading at k gives v
    np.testing.assert_allclose(o, v, rtol=1e-5)
    # the matrix form S2 = (I - beta k k^T) g S + beta k v^T
    S3, o3 = orc.delta_step(S, v.repeat(2)[:6], k, v, 0.7, 0.4)
    np.testing.assert_allclose(S3, (np.eye(6) - 0.4 * np.outer(k, k)) @ (0.7 * S) + 0.4 * np.outer(k, v), rtol=1e-12)
    np.testing.assert_allclose(o3, S3.T @ v.repeat(2)[:6])


def test_gla_equals_its_attention_form():
    g = np.random.default_rng(2)
    T, d, e = 9, 5, 3
    q, k, v = g.standard_normal((T, d)), g.standard_normal((T, d)), g.standard_normal((T, e))
    a = orc.gla_decay(g.standard_normal((T, d)), 3.0)
    S, out = np.zeros((d, e)), []
    for t in range(T):
        S, o = orc.gla_step(S, q[t], k[t], v[t], a[t])
        out.append(o)
    c = np.cumsum(np.log(a), 0)
    for t in range(T):
        w = [np.sum(q[t] * k[j] * np.exp(c[t] - c[j])) for j in range(t + 1)]
        np.testing.assert_allclose(out[t], w @ v[:t + 1], rtol=1e-9)


def test_short_convolution_and_decays():
    g = np.random.default_rng(3)
    x, taps = g.standard_normal((7, 2)), g.standard_normal((2, 3))
    for c in range(2):
        full = np.convolve(np.concatenate([[0, 0], x[:, c]]), taps[c][::-1], "valid")
        for t in range(7):
            window = np.concatenate([np.zeros((2, 2)), x])[t:t + 3]
            assert abs(orc.short_conv(window, taps)[c] - orc.silu(full[t])) < 1e-12
    assert abs(orc.delta_decay(0.3, 0.5, -0.1) - np.exp(-np.exp(0.5) * np.log1p(np.exp(0.2)))) < 1e-12
    assert orc.chunk_start(9, 5) == 5 and orc.chunk_start(10, 5) == 10 and orc.chunk_start(4, 5) == 0


def test_chunks_and_state_in_the_oracle():
    """Outside its chunk a token reaches a later one only through the recurrences."""
    g = np.random.default_rng(4)
    w = {n: g.standard_normal(s) / np.sqrt(max(1, s[-1] if s else 1)) for n, s in synth.stack_tensor_shapes(CFG, 3).items()}
    ids = [1, 2, 3, 4, 5, 6, 7]
    m = orc.Model(CFG, w)
    whole = m.run(ids)
    st = m.new_state()
    parts = np.concatenate([m.run(ids[:3], st), m.run(ids[3:], st)])
    np.testing.assert_array_equal(whole, parts)
    quiet = dict(w, **{n: np.zeros_like(a) for n, a in w.items() if n.endswith("right.o") or n == "l1.mix.o"})
    a, b = orc.Model(CFG, quiet).run(ids), orc.Model(CFG, quiet).run([9] + ids[1:])
    assert np.abs(a[4] - b[4]).max() > 1e-6 and np.abs(a[5] - b[5]).max() == 0.0


def write(tmp_path, cfg, drop=(), rank=3):
    tensors = {n: np.zeros(s, np.float32) for n, s in synth.stack_tensor_shapes(CFG, rank).items() if n not in drop}
    synth.write_model_dir(tmp_path, cfg, tensors.items())
    return tmp_path


@pytest.mark.parametrize("path,value,message", [
    ("architecture", "Nowhere", "unknown architecture `Nowhere`"),
    ("vocab", 0, "vocab must be an integer"),
    ("width", None, "missing field `width`"),
    ("logit_scale", 0, "logit_scale must not be 0"),
    ("norm.eps", "small", "norm.eps must be a finite number"),
    ("layers", [], "must be a list"),
    ("layers.0.type", "conv", r"layers\[0\] type `conv` is not supported"),
    ("layers.0.mixer.left.vdim", 4, "the values are the keys"),
    ("layers.0.mixer.left.kv_heads", 3, "heads must be a multiple of kv_heads"),
    ("layers.0.mixer.left.rot.dims", 3, "dims must be even"),
    ("layers.0.mixer.left.rot.dims", 8, "rot.dims must be an integer in"),
    ("layers.0.mixer.left.mask.size", 0, "mask.size must be an integer"),
    ("layers.0.mixer.right.conv", 99, "conv must be an integer"),
    ("layers.0.mixer.right", None, r"missing field `layers\[0\].mixer.right`"),
    ("layers.0.mlp.kind", "experts", "kind `experts` is not supported"),
    ("layers.1.mixer.tau", 0.0, "tau must be > 0"),
])
def test_config_errors(tmp_path, path, value, message):
    cfg = copy.deepcopy(CFG)
    node, *keys = [cfg] + path.split(".")
    for k in keys[:-1]:
        node = node[int(k)] if k.isdigit() else node[k]
    if value is None:
        del node[keys[-1]]
    else:
        node[keys[-1]] = value
    with pytest.raises(Gpt2Error, match=message):
        load_model(write(tmp_path, cfg))


def test_asset_errors(tmp_path):
    with pytest.raises(Gpt2Error, match="failed to read config"):
        load_model(tmp_path)
    (tmp_path / "config.json").write_text("[]")
    with pytest.raises(Gpt2Error, match="expected an object"):
        load_model(tmp_path)
    (tmp_path / "config.json").write_text(json.dumps(CFG))
    with pytest.raises(Gpt2Error, match="failed to read safetensors file"):
        load_model(tmp_path)
    with pytest.raises(Gpt2Error, match="l1.mix.a1"):
        load_model(write(tmp_path, CFG, drop=("l1.mix.a1",)))


def test_model_without_a_device_or_with_one(tmp_path, has_gpu):
    if has_gpu:
        with pytest.raises(Gpt2Error, match="tensor `l0.mix.left.pb` not found"):
            load_model(write(tmp_path, CFG, drop=("l0.mix.left.pb",)))
    else:
        with pytest.raises(Gpt2Error, match="no HIP device"):
            load_model(write(tmp_path, CFG))
