"""CPU-only: the Movudra oracle's mechanisms in other forms than its own loops, and the errors of the
config reader before any device work."""
import copy

import numpy as np
import pytest

import oracle.movudra as orc
from puppygrad_amd import Gpt2Error, load_model, synth

YARN = {"factor": 4.0, "original": 50, "fast": 6.0, "slow": 1.0}
CFG = {"architecture": "Movudra", "vocab": 19, "width": 20, "norm": {"eps": 1e-5}, "layers": [
    {"type": "mamba2", "mlp": {"kind": "dense", "ff": 12},
     "mixer": {"heads": 4, "vdim": 6, "state": 5, "groups": 2, "norm_groups": 3, "conv": 3}},
    {"type": "latent_attention", "mlp": {"kind": "moe", "router": {"experts": 4, "top": 2}, "expert": {"ff": 7}},
     "mixer": {"heads": 2, "dim": 6, "rot_dim": 4, "vdim": 5, "kv_rank": 9, "q_rank": 8, "mask": {"size": 4}, "scale": 0.3,
               "rot": {"dims": 4, "base": 100.0, "scaling": YARN}}},
    {"type": "channel_delta", "mlp": None, "mixer": {"heads": 4, "kv_heads": 2, "dim": 4, "vdim": 6, "conv": 2}}]}
RANKS = (3, 2)


def random_weights(seed):
    g = np.random.default_rng(seed)
    return {n: g.standard_normal(s) / np.sqrt(s[-1]) for n, s in synth.stack_tensor_shapes(CFG, RANKS).items()}


def test_rotation():
    g = np.random.default_rng(0)
    q, k = g.standard_normal(10), g.standard_normal(10)
    for scaling in (None, YARN):
        f, mag = orc.yarn_frequencies(6, 30.0, scaling)
        dots = [orc.rotate_pairs(q, p + 7, f, mag) @ orc.rotate_pairs(k, p, f, mag) for p in (0, 3, 1000)]
        np.testing.assert_allclose(dots, dots[0], rtol=1e-9)
        # the complex form: value 2 i + j value 2 i + 1 times mag exp(j p f_i)
        z = (q[0:6:2] + 1j * q[1:6:2]) * mag * np.exp(5j * np.array(f))
        got = orc.rotate_pairs(q, 5, f, mag)
        np.testing.assert_allclose(got[0:6:2] + 1j * got[1:6:2], z, rtol=1e-12)
        np.testing.assert_array_equal(got[6:], q[6:])


def test_yarn_keeps_fast_pairs_and_stretches_slow_ones():
    plain, one = orc.yarn_frequencies(64, 10000.0, None)
    f, mag = orc.yarn_frequencies(64, 10000.0, {"factor": 8.0, "original": 2000, "fast": 30.0, "slow": 1.0})
    r = np.array(f) / plain
    assert one == 1.0 and abs(mag - (0.1 * np.log(8.0) + 1.0)) < 1e-12
    turns = 2000 * np.array(plain) / (2 * np.pi)
    assert (r[turns > 40] == 1.0).all() and np.allclose(r[turns < 0.7], 1 / 8.0)
    assert (np.diff(r) <= 1e-12).all() and ((r > 0.13) & (r < 0.99)).any()


def test_sink_attention():
    g = np.random.default_rng(1)
    q, keys, values = g.standard_normal(4), g.standard_normal((6, 4)), g.standard_normal((6, 3))
    # the sink is a key of its own with score `sink` and value 0
    z = np.append(keys @ q * 0.7, 1.3)
    w = orc.softmax(z)
    np.testing.assert_allclose(orc.sink_attention(q, keys, values, 0.7, 1.3), w[:6] @ values, rtol=1e-12)
    assert orc.window_start(9, 4) == 6 and orc.window_start(2, 4) == 0 and orc.window_start(5, 1) == 5


def test_ssd_equals_its_attention_form():
    g = np.random.default_rng(2)
    T, N, e, a = 9, 5, 3, -0.7
    B, C, x, dt = g.standard_normal((T, N)), g.standard_normal((T, N)), g.standard_normal((T, e)), g.uniform(0.1, 1.0, T)
    S, out = np.zeros((N, e)), []
    for t in range(T):
        S, o = orc.ssd_step(S, a, dt[t], B[t], C[t], x[t])
        out.append(o)
    G = np.cumsum(a * dt)
    for t in range(T):
        w = np.array([C[t] @ B[j] * np.exp(G[t] - G[j]) * dt[j] for j in range(t + 1)])
        np.testing.assert_allclose(out[t], w @ x[:t + 1], rtol=1e-9)


def test_channel_delta_rule():
    g = np.random.default_rng(3)
    k, v, q = orc.unit(g.standard_normal(6)), g.standard_normal(4), g.standard_normal(6)
    S, a = g.standard_normal((6, 4)), g.uniform(0.2, 1.0, 6)
    S2, o = orc.channel_delta_step(S, q, k, v, a, 0.4)
    np.testing.assert_allclose(S2, (np.eye(6) - 0.4 * np.outer(k, k)) @ np.diag(a) @ S + 0.4 * np.outer(k, v), rtol=1e-12)
    np.testing.assert_allclose(o, S2.T @ q)
    _, o = orc.channel_delta_step(S, k, k, v, np.ones(6), 1.0)
    np.testing.assert_allclose(o, v, rtol=1e-5)


def test_routing_and_group_norm():
    chosen, w = orc.route(np.array([0.0, 2.0, 1.0, 2.0]), 3)
    assert chosen.tolist() == [1, 3, 2] and abs(w[0] - np.exp(2) / (1 + 2 * np.exp(2) + np.e)) < 1e-12 and w.sum() < 1.0
    y = np.arange(1.0, 13.0)
    got = orc.group_rms(y, 3, 0.5)
    np.testing.assert_allclose(got[4:8], y[4:8] / np.sqrt(np.mean(y[4:8] ** 2) + 0.5))


def test_windows_and_state_in_the_oracle():
    """Beyond its window a token reaches a later one only through the recurrences."""
    w = random_weights(4)
    ids = [1, 2, 3, 4, 5, 6, 7]
    m = orc.Model(CFG, w)
    whole = m.run(ids)
    st = m.new_state()
    np.testing.assert_array_equal(whole, np.concatenate([m.run(ids[:3], st), m.run(ids[3:], st)]))
    quiet = dict(w, **{n: np.zeros_like(w[n]) for n in ("l0.mix.o", "l2.mix.o")})
    a, b = orc.Model(CFG, quiet).run(ids), orc.Model(CFG, quiet).run([9] + ids[1:])
    assert np.abs(a[3] - b[3]).max() > 1e-6 and np.abs(a[4] - b[4]).max() == 0.0


def write(tmp_path, cfg, drop=(), **other):
    tensors = {n: np.zeros(s, np.float32) for n, s in synth.stack_tensor_shapes(CFG, RANKS).items() if n not in drop}
    tensors.update({n.replace("__", "."): np.zeros(s, np.float32) for n, s in other.items()})
    synth.write_model_dir(tmp_path, cfg, tensors.items())
    return tmp_path


@pytest.mark.parametrize("path,value,message", [
    ("architecture", "Nowhere", "unknown architecture `Nowhere`"),
    ("vocab", 0, "vocab must be an integer"),
    ("norm", None, "missing field `norm`"),
    ("layers.0.type", "gla", r"layers\[0\] type `gla` is not supported"),
    ("layers.0.mlp.kind", "gated", "kind `gated` is not supported"),
    ("layers.0.mlp.ff", 0, "ff must be an integer"),
    ("layers.0.mixer.groups", 3, "heads must be a multiple of groups"),
    ("layers.0.mixer.norm_groups", 5, "multiple of norm_groups"),
    ("layers.0.mixer.state", 300, "state must be an integer in"),
    ("layers.0.mixer.conv", 99, "conv must be an integer"),
    ("layers.1.mixer.rot.dims", 3, "dims must be even"),
    ("layers.1.mixer.rot.dims", 8, "rot.dims must be an integer in"),
    ("layers.1.mixer.rot.scaling.factor", None, "missing field"),
    ("layers.1.mixer.rot.scaling.slow", 0.0, "must hold numbers > 0"),
    ("layers.1.mixer.dim", 254, "dim . rot_dim may be up to"),
    ("layers.1.mixer.mask", None, "missing field"),
    ("layers.1.mixer.scale", "big", "scale must be a finite number"),
    ("layers.1.mlp.router.top", 5, "top must be an integer"),
    ("layers.1.mlp.router.experts", None, "missing field"),
    ("layers.2.mixer.kv_heads", 3, "heads must be a multiple of kv_heads"),
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


def test_asset_errors(tmp_path, has_gpu):
    with pytest.raises(Gpt2Error, match="l2.mix.g1"):
        load_model(write(tmp_path, CFG, drop=("l2.mix.g1",)))
    with pytest.raises(Gpt2Error, match="l2.mix.a1 must have two dimensions"):
        load_model(write(tmp_path, CFG, l2__mix__a1=(3,)))
    if has_gpu:
        with pytest.raises(Gpt2Error, match="tensor `l1.mlp.e3.up` not found"):
            load_model(write(tmp_path, CFG, drop=("l1.mlp.e3.up",)))
        with pytest.raises(Gpt2Error, match="does not match expected"):
            load_model(write(tmp_path, CFG, l1__mix__sink=(3,)))
    else:
        with pytest.raises(Gpt2Error, match="no HIP device"):
            load_model(write(tmp_path, CFG))


def test_benchmark_sizes_have_equal_layers():
    """What a token meets in a layer is 12 width^2 parameters, within 2 %."""
    for width in synth.MOVUDRA_SIZES:
        cfg = synth.movudra_config(width, 4)
        shapes = synth.stack_tensor_shapes(cfg)
        for i, layer in enumerate(cfg["layers"]):
            n = sum(int(np.prod(s)) for name, s in shapes.items() if name.startswith(f"l{i}."))
            if layer["mlp"]["kind"] == "moe":
                n -= 3 * (synth.MOVUDRA_EXPERTS - synth.MOVUDRA_TOP) * layer["mlp"]["expert"]["ff"] * width
            assert abs(n / (12 * width * width) - 1) < 0.02, (width, i)
