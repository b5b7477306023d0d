"""Movudra on the GPU against the plain float64 oracle (oracle/movudra.py): every mechanism alone,
prompts, portions, decoding through the cache, batches, reused caches, window edges, other sizes,
generation and the trace runner.  Configurations and weights are made here."""
import os

import numpy as np
import pytest

import oracle.movudra as orc
from puppygrad_amd import (Gpt2Error, Gpt2HipConfig, LogitsSampler, StackModel, TextGenerationConfig, _lib, generate,
                           load_model, synth)
from stack_helpers import Pair as AnyPair, check, ref_greedy, rounded, run_trace, same_until_close

pytestmark = pytest.mark.gpu
BF16, F32 = _lib.PG_STORE_BF16, _lib.PG_STORE_F32
YARN = {"factor": 6.0, "original": 60, "fast": 8.0, "slow": 1.0}


class Pair(AnyPair):
    def __init__(self, *args, **kw):
        super().__init__(orc, *args, **kw)


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def moe(experts=7, top=2, ff=24):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def mamba(heads=6, vdim=8, state=12, groups=2, norm_groups=3, conv=4, mlp=None):
    return {"type": "mamba2", "mlp": mlp, "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
                                                    "norm_groups": norm_groups, "conv": conv}}


def delta(heads=4, kv=2, dim=8, vdim=12, conv=3, mlp=None):
    return {"type": "channel_delta", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}}


def latent(heads=4, dim=16, rot=8, vdim=12, kv=20, q=24, window=12, base=500.0, scaling=YARN, scale=None, mlp=None):
    return {"type": "latent_attention", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": kv, "q_rank": q, "mask": {"size": window},
        "scale": (dim + rot) ** -0.5 if scale is None else scale, "rot": {"dims": rot, "base": base, "scaling": scaling}}}


def config(layers, width=48, vocab=61, eps=1e-5):
    return {"architecture": "Movudra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


MIXED = config([delta(mlp=moe()), latent(mlp=dense()), mamba(mlp=moe(5, 3, 20)), latent(3, 24, 6, 20, 33, 17, 19),
                mamba(4, 11, 8, 4, 1, 2), delta(6, 3, 20, 16, 4, mlp=dense(33))])


def weights(cfg, seed, ranks=(5, 3), **fixed):
    """Random weights of order-one activations; `fixed` replaces tensors (dots in names as __)."""
    g = np.random.default_rng(seed)
    out = {}
    for name, shape in synth.stack_tensor_shapes(cfg, ranks).items():
        last = name.split(".")[-1]
        if last.startswith("norm"):
            a = 1.0 + 0.2 * g.standard_normal(shape)
        elif last in ("dt_bias", "sink", "D"):
            a = g.standard_normal(shape)
        elif last == "b" and len(shape) == 1:
            a = 0.3 * g.standard_normal(shape)
        elif last == "A_log":
            a = g.uniform(-2.0, 1.0, shape)
        elif last == "conv":
            a = 0.6 * g.standard_normal(shape)
        elif last == "embed":
            a = g.standard_normal(shape)
        elif last == "router":
            a = 3.0 * g.standard_normal(shape) / np.sqrt(shape[-1])
        else:
            a = g.standard_normal(shape) / np.sqrt(shape[-1])
        out[name] = a
    for name, a in fixed.items():
        name = name.replace("__", ".")
        assert out[name].shape == np.shape(a), name
        out[name] = a
    return rounded(out)


@pytest.fixture(scope="module")
def mixed(tmp_path_factory):
    return Pair(tmp_path_factory.mktemp("mixed"), MIXED, weights(MIXED, 11))


def all_ways(p, ids, portions=((2, 3, 1, 33, 2),), tol=2e-5):
    want = p.ref.run(ids)
    check(p.portions(ids, [len(ids)]), want, tol, what="prompt")
    check(p.portions(ids, [1]), want, tol, what="decoded")
    for sizes in portions:
        check(p.portions(ids, list(sizes)), want, tol, what=f"portions {sizes}")
    return want


# ---- mechanisms ------------------------------------------------------------------------------------
@pytest.mark.parametrize("storage", [BF16, F32], ids=["bf16", "f32"])
@pytest.mark.parametrize("layer", [
    mamba(), mamba(conv=1), mamba(6, 8, 12, 2, 4), mamba(4, 8, 16, 1, 1, 2), mamba(3, 5, 7, 3, 5, 3), mamba(2, 64, 128, 1, 2),
    mamba(2, 128, 64, 2, 1, 6), mamba(1, 1, 1, 1, 1, 2), mamba(2, 200, 160, 1, 8), mamba(1, 256, 256, 1, 1), mamba(12, 20, 96, 4, 12)],
    ids=["base", "taps1", "parts-across-heads", "one-group", "odd", "n128", "v128", "ones", "n160", "n256", "n96"])
def test_mamba2_alone(tmp_path, layer, storage):
    cfg = config([layer])
    p = Pair(tmp_path, cfg, weights(cfg, 3), storage)
    all_ways(p, p.ids(75))


@pytest.mark.parametrize("layer,ranks", [
    (delta(), (5, 3)), (delta(3, 3, 16, 16, 1), (1, 1)), (delta(4, 1, 20, 40, 2), (33, 40)), (delta(2, 1, 64, 128, 4), (16, 64)),
    (delta(2, 2, 128, 64, 6), (70, 8)), (delta(1, 1, 4, 3, 4), (2, 2)), (delta(2, 1, 160, 200, 3), (24, 24)),
    (delta(1, 1, 256, 256, 4), (24, 32)), (delta(1, 1, 1, 1, 2), (1, 1)), (delta(4, 2, 96, 30, 3), (32, 31))],
    ids=["base", "taps1", "ranks", "vdim128", "taps6", "tiny", "d160", "d256", "ones", "d96"])
@pytest.mark.parametrize("storage", [BF16, F32], ids=["bf16", "f32"])
def test_channel_delta_alone(tmp_path, layer, ranks, storage):
    cfg = config([layer])
    p = Pair(tmp_path, cfg, weights(cfg, 4, ranks), storage)
    all_ways(p, p.ids(75))


@pytest.mark.parametrize("layer", [
    latent(), latent(scaling=None), latent(window=1), latent(3, 5, 6, 7, 33, 17, 9), latent(1, 4, 2, 4, 8, 3, 33),
    latent(17, 64, 32, 48, 100, 40, 70), latent(2, 128, 64, 128, 512, 96, 40), latent(2, 192, 64, 256, 600, 70, 33),
    latent(2, 30, 2, 130, 1024, 10, 200), latent(4, 24, 0, 20, 32, 32, 21), latent(5, 60, 4, 64, 64, 64, 150, base=20.0),
    latent(2, 100, 28, 32, 40, 20, 64, scaling={"factor": 40.0, "original": 4096, "fast": 32.0, "slow": 1.0}, base=10000.0)],
    ids=["base", "plain-rotation", "window1", "odd", "one-head", "heads17", "d192", "d256", "rank1024", "unrotated", "d64", "d128"])
@pytest.mark.parametrize("storage", [BF16, F32], ids=["bf16", "f32"])
def test_latent_attention_alone(tmp_path, layer, storage):
    cfg = config([layer])
    p = Pair(tmp_path, cfg, weights(cfg, 5), storage)
    all_ways(p, p.ids(150), ((50, 1, 1, 1, 7, 2, 40, 1, 2), (2,)))


def test_partly_rotated_part(tmp_path):
    layer = latent(rot=12)
    layer["mixer"]["rot"]["dims"] = 6
    cfg = config([layer])
    p = Pair(tmp_path, cfg, weights(cfg, 6))
    all_ways(p, p.ids(60))


def test_large_scores_and_sinks(tmp_path):
    """Sinks that take almost everything or nothing, beside scores of order 100."""
    cfg = config([latent(6, window=24, scale=20.0), latent(6, window=24)])
    w = weights(cfg, 8, l0__mix__sink=[-200.0, 300.0, 0.0, -3.0, 40.0, 9.0], l1__mix__sink=[-200.0, 200.0, 0.0, -3.0, 4.0, 9.0])
    p = Pair(tmp_path, cfg, w)
    all_ways(p, p.ids(60), tol=1e-4)
    # the sink shows
    other = orc.Model(cfg, dict(w, **{"l1.mix.sink": np.full(6, -50.0)})).run(p.ids(20))
    assert np.abs(other - p.ref.run(p.ids(20))).max() > 0.05


@pytest.mark.parametrize("mlp", [dense(1), dense(33), dense(200), moe(1, 1, 8), moe(5, 5, 24), moe(70, 3, 16), moe(300, 8, 8),
                                 moe(12, 1, 33), moe(2, 2, 100), moe(1024, 64, 4)],
                         ids=["ff1", "ff33", "ff200", "one", "all", "e70", "e300", "top1", "e2", "top64"])
@pytest.mark.parametrize("storage", [BF16, F32], ids=["bf16", "f32"])
def test_feed_forward_and_norms_alone(tmp_path, mlp, storage):
    cfg = config([delta(1, 1, 4, 4, 2, mlp=mlp)], width=37, eps=0.3)
    p = Pair(tmp_path, cfg, weights(cfg, 17), storage)  # (a seed without equal logits at the last place)
    all_ways(p, p.ids(150), ((40, 3, 1, 20, 2),))


def test_experts_of_unequal_load(tmp_path):
    """Most rows at one expert and some experts without any, in tiles of both sizes."""
    cfg = config([mamba(mlp=moe(6, 2, 40)), mamba(mlp=moe(3, 1, 40))], width=64)
    w = weights(cfg, 9)
    w["l0.mlp.router"][4] *= 0.0
    w["l1.mlp.router"][:2] *= 0.01
    p = Pair(tmp_path, cfg, rounded(w))
    all_ways(p, p.ids(420), ((300, 33, 87),))


@pytest.mark.parametrize("storage", [BF16, F32], ids=["bf16", "f32"])
def test_experts_of_many_rows(tmp_path, storage):
    """Enough rows for the largest tiles of an expert."""
    cfg = config([mamba(4, 16, 8, 1, 1, 2, mlp=moe(2, 1, 70)), mamba(4, 16, 8, 1, 1, 2, mlp=moe(4, 3, 9))], width=100)
    p = Pair(tmp_path, cfg, weights(cfg, 10), storage)
    ids = p.ids(1100)
    check(p.portions(ids, [1100]), p.ref.run(ids))


def test_strong_decays(tmp_path):
    """Decays from none to a state that is wiped by a single token, side by side."""
    cfg = config([mamba(), delta(), delta(2, 2, 32, 16)])
    w = weights(cfg, 6)
    w["l0.mix.A_log"] = np.linspace(-8, 4, 6)
    w["l1.mix.A_log"] = np.linspace(-8, 4, 4)
    w["l2.mix.A_log"] = np.array([3.0, 0.0])
    for i in (1, 2):
        n = w[f"l{i}.mix.dt_bias"].shape[0]
        w[f"l{i}.mix.dt_bias"] = np.random.default_rng(i).permutation(np.linspace(-12, 30, n))
        w[f"l{i}.mix.a2"] *= 4
    p = Pair(tmp_path, cfg, rounded(w))
    all_ways(p, p.ids(140))


def test_old_state(tmp_path):
    """A write at the first token that nothing decays is still read hundreds of tokens later."""
    cfg = config([mamba(1, 8, 8, 1, 1, 2), delta(1, 1, 8, 8, 2)], width=24, vocab=16)
    w = weights(cfg, 70)
    w["l0.mix.A_log"] = np.full(1, -9.0)
    w["l1.mix.A_log"] = np.full(1, -9.0)
    w["l1.mix.b"] = w["l1.mix.b"] * 0.1 - 0.2
    p = Pair(tmp_path, cfg, rounded(w))
    base = p.ids(400, seed=9)
    for first in (1, 2):
        ids = [first] + base[1:]
        want = p.ref.run(ids)
        check(p.portions(ids, [400]), want, 1e-4)
        check(p.portions(ids, [200, 1]), want, 1e-4)
    a, b = p.ref.run([1] + base[1:])[-1], p.ref.run([2] + base[1:])[-1]
    assert np.abs(a - b).max() > 1e-3 * np.abs(a).max()  # (the first token shows)


def test_far_rotations(tmp_path):
    """Angles of positions in the thousands."""
    cfg = config([latent(2, 8, 8, 8, 16, 16, 40, scaling=None), latent(2, 8, 8, 8, 16, 16, 40)], width=24, vocab=30)
    p = Pair(tmp_path, cfg, weights(cfg, 71))
    ids = p.ids(3000)
    want = p.ref.run(ids)[-50:]
    cache = p.dev.new_kv_cache()
    p.dev.extend(ids[:2950], cache, [])
    got = [p.dev.extend(ids[2950:2980], cache, range(30)).to_host().reshape(30, -1)]
    got += [p.dev.forward_one(t, cache).to_host()[None] for t in ids[2980:]]
    check(np.concatenate(got), want)


# ---- whole models ----------------------------------------------------------------------------------
@pytest.mark.parametrize("storage", [BF16, F32], ids=["bf16", "f32"])
@pytest.mark.parametrize("width", [48, 50, 33, 160])
def test_prompt_portions_and_decoding(tmp_path, width, storage):
    cfg = dict(MIXED, width=width)
    p = Pair(tmp_path, cfg, weights(cfg, 20 + width), storage)
    all_ways(p, p.ids(101), ([2], [3], [7], [16], [31], [32], [33], [64], [90, 1], [1, 2, 3, 5, 8, 13, 21, 34]),
             tol=5e-5)  # (six layers of rounding)


def test_layer_order_and_first_layers(tmp_path):
    for i, layers in enumerate(([latent()], [mamba(mlp=moe())], [delta(), delta(mlp=dense()), latent(mlp=moe())],
                                [latent(mlp=dense()), mamba(), latent(mlp=moe(4, 1, 8))])):
        cfg = config(layers)
        p = Pair(tmp_path / str(i), cfg, weights(cfg, 30 + i))
        all_ways(p, p.ids(45), ((11, 1),))


def test_mixers_of_unequal_width(tmp_path):
    """What a wide mixer leaves behind the columns of a narrow one is not part of the narrow one's norm."""
    for i, groups in enumerate((1, 2, 3, 6)):
        cfg = config([latent(4, 16, 8, 40), mamba(6, 7, 8, 2, groups), delta(4, 2, 8, 30), mamba(6, 5, 8, 2, groups, mlp=dense(7))])
        p = Pair(tmp_path / str(i), cfg, weights(cfg, 35 + i))
        all_ways(p, p.ids(40), ((11, 1),))


def test_first_tokens(mixed):
    for n in (1, 2, 3, 4, 5):
        ids = mixed.ids(n, seed=40 + n)
        want = mixed.ref.run(ids)
        check(mixed.portions(ids, [n]), want, what=f"{n} tokens")
        check(mixed.portions(ids, [1]), want, what=f"{n} tokens decoded")
        cache = mixed.dev.new_kv_cache()
        check(mixed.dev.prefill(ids, cache).to_host(), want[-1])


def test_forward_matches_prefill_and_wanted_places(mixed):
    ids = mixed.ids(70, seed=3)
    want = mixed.ref.run(ids)
    check(mixed.dev.forward(ids).logits, want)
    cache = mixed.dev.new_kv_cache()
    check(mixed.dev.prefill(ids[:-1], cache).to_host(), want[-2])
    check(mixed.dev.forward_one(ids[-1], cache).to_host(), want[-1])
    cache.clear()
    assert mixed.dev.extend(ids[:20], cache, []) is None
    check(mixed.dev.extend(ids[20:40], cache, [0, 3, 19]).to_host(), want[[20, 23, 39]])


def test_long_prompt_in_internal_segments(tmp_path):
    """More tokens than one pass over the layers takes."""
    cfg = config([latent(1, 4, 2, 4, 8, 8, 50), mamba(1, 4, 4, 1, 1, 2), delta(1, 1, 4, 4, 2, mlp=moe(3, 1, 4))], width=8, vocab=11)
    p = Pair(tmp_path, cfg, weights(cfg, 50))
    ids = p.ids(8192 + 75)
    want = p.ref.run(ids)[-80:]
    cache = p.dev.new_kv_cache()
    check(p.dev.extend(ids, cache, range(len(ids) - 80, len(ids))).to_host(), want, 1e-4)


def test_long_decoding(mixed):
    ids = mixed.ids(330, seed=5)
    check(mixed.portions(ids, [10, 1]), mixed.ref.run(ids))


# ---- batches, reused caches ------------------------------------------------------------------------
@pytest.mark.parametrize("batch", [2, 5, 33])  # (33: more pairs of rows and experts than go one by one)
def test_batch_against_each_alone(mixed, batch):
    T, steps = 21, 16
    ids = np.array([mixed.ids(T + steps, seed=100 + b) for b in range(batch)])
    cache = mixed.dev.new_kv_cache(batch)
    for _ in range(2):  # (the second time over what the first left)
        got = [mixed.dev.prefill_batch(ids[:, :T], cache).to_host()]
        for t in range(T, T + steps):
            got.append(mixed.dev.forward_one_batch(ids[:, t], cache).to_host())
        got = np.stack(got, 1)
        for b in (0, 1, batch - 1):
            check(got[b], mixed.ref.run(ids[b])[T - 1:], what=f"sequence {b}")


def test_requests_of_unequal_length_side_by_side(mixed):
    lens = (3, 40, 17)
    ids = [mixed.ids(n, seed=60 + n) for n in lens]
    want = [mixed.ref.run(i) for i in ids]
    caches, at = [mixed.dev.new_kv_cache() for _ in lens], [0] * 3
    for k in range(60):
        i = k % 3
        n = min((1, 5, 2)[i], lens[i] - at[i])
        if n:
            got = mixed.dev.extend(ids[i][at[i]:at[i] + n], caches[i], range(n)).to_host().reshape(n, -1)
            check(got, want[i][at[i]:at[i] + n], what=f"request {i} at {at[i]}")
            at[i] += n
    assert at == list(lens)


def test_cache_used_again(mixed):
    """Sequences one after the other in one cache, in all ways to start, and rewinding."""
    cache = mixed.dev.new_kv_cache()
    long = mixed.ids(80, seed=6)
    for k, n in enumerate((33, 2, 1, 60, 5)):
        mixed.portions(long, [80], cache)
        ids = mixed.ids(n, seed=300 + k)
        check(mixed.portions(ids, [n] if k % 2 else [1], cache), mixed.ref.run(ids))
    with pytest.raises(Gpt2Error, match="cannot be set back"):
        cache.seq_len = 3
    cache.seq_len = 0
    check(mixed.dev.forward_one(7, cache).to_host(), mixed.ref.run([7])[-1])


# ---- keys that stand out ---------------------------------------------------------------------------
def beacon_model(tmp_path, window, heads=2, strength=6.0):
    """One latent attention in which the query of token 1 meets the key of token 2 with a score of
    about 30 and everything else with about 0."""
    layer = latent(heads, 6, 4, 6, 8, 4, window, scale=1.0)
    cfg = config([layer], width=32, vocab=32)
    g = np.random.default_rng(1)
    w = weights(cfg, 60)
    embed = np.zeros((32, 32))
    embed[np.arange(32), np.arange(32)] = 4.0
    dkv = g.standard_normal((12, 32))
    dkv[7], dkv[:7, 2], dkv[8:] = 0.0, 0.0, 0.1 * dkv[8:]
    dkv[7, 2] = 1.0                       # token 2 alone has the last latent value
    dq = np.zeros((4, 32))
    dq[1], dq[0, 1], dq[1, 1] = 1.0, 1.0, 0.0
    uq, uk = np.zeros((heads, 10, 4)), np.zeros((heads, 6, 8))
    uq[:, 5, 0] = strength
    uk[:, 5, 7] = 1.0
    w.update({"embed": embed, "l0.mix.dkv": dkv, "l0.mix.dq": dq, "l0.mix.uq": uq.reshape(-1, 4),
              "l0.mix.uk": uk.reshape(-1, 8), "l0.mix.dq.norm": np.ones(4), "l0.mix.dkv.norm": np.ones(8),
              "l0.mix.sink": np.full(heads, 2.0)})
    return Pair(tmp_path, cfg, rounded(w))


@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 64, 65, 96, 128, 257])
def test_key_inside_and_outside_the_window(tmp_path, window):
    p = beacon_model(tmp_path, window)
    n = 2 * window + 40
    fill = [3 + i % 20 for i in range(n)]
    cache = p.dev.new_kv_cache()
    for query in sorted({window - 1, window, window + 1, 2 * window, n - 1}):
        for back in sorted({1, window // 2, window - 1, window, window + 1}):
            key = query - back
            if back < 1 or key < 0:
                continue
            ids = fill[:query + 1]
            ids[key], ids[query] = 2, 1
            want = p.ref.run(ids)[-1]
            without = list(ids)
            without[key] = 3
            gap = np.sqrt(np.mean((want - p.ref.run(without)[-1]) ** 2)) / np.sqrt(np.mean(want ** 2))
            assert gap > 0.05 if back < window else gap < 1e-9, (key, query, gap)  # whether the key is seen shows
            cache.clear()
            check(p.dev.prefill(ids, cache).to_host(), want, what=f"prompt {key} {query}")
            cache.clear()
            p.dev.extend(ids[:-1], cache, [])
            check(p.dev.forward_one(1, cache).to_host(), want, what=f"decoded {key} {query}")
            if query >= 3:
                cache.clear()
                p.dev.extend(ids[:-2], cache, [])
                check(p.dev.extend(ids[-2:], cache).to_host(), want, what=f"two tokens {key} {query}")


def test_every_key_of_a_window_is_found(tmp_path):
    """One standing-out key at each place of a window of several shares, decoded and in portions."""
    window = 150
    p = beacon_model(tmp_path, window, heads=3)
    cache = p.dev.new_kv_cache()
    fill = [3 + i % 20 for i in range(2 * window + 9)]
    for back in list(range(1, window, 7)) + [15, 16, 31, 32, 63, 64, 127, 128, window - 1]:
        ids = list(fill)
        ids[len(ids) - 1 - back], ids[-1] = 2, 1
        want = p.ref.run(ids[-window - 1:])[-1]  # (nothing but the window is seen, and only distances count)
        cache.clear()
        p.dev.extend(ids[:-1], cache, [])
        check(p.dev.forward_one(1, cache).to_host(), want, 1e-4, what=f"{back} back")
        cache.clear()
        p.dev.extend(ids[:-40], cache, [])
        check(p.dev.extend(ids[-40:], cache).to_host(), want, 1e-4, what=f"{back} back, portion")


# ---- generation ------------------------------------------------------------------------------------
@pytest.mark.parametrize("path", [_lib.PG_DECODE_AUTO, _lib.PG_DECODE_KERNELS], ids=["graph", "kernels"])
def test_greedy_generation(tmp_path, path):
    p = Pair(tmp_path, MIXED, weights(MIXED, 11), decode_path=path)
    ids, n = p.ids(14, seed=10), 60
    want, gaps = ref_greedy(p, ids, n)
    cache = p.dev.new_kv_cache()
    for _ in range(3):  # (the one-token step is captured on the way: every replay must agree)
        p.dev.prefill(ids, cache)
        got, stats = p.dev.decode_greedy(cache, n)
        assert len(got) == n and stats.generated_tokens == n and cache.seq_len == len(ids) + n - 1
        assert same_until_close(got, want, gaps) > 20
        p.dev.forward_one(got[-1], cache)  # eager work between the replays
    assert generate(p.dev, ids, 20, lambda _t: None)[14:] == got[:20]
    assert p.dev.generate_greedy_cached(ids, 20)[14:] == got[:20]
    assert p.dev.generate_greedy(ids, 12)[14:] == got[:12]
    out, stats = p.dev.stream_token_ids_with_stats(ids, TextGenerationConfig(25))
    assert out == ids + got[:25] and stats.prompt_tokens == 14
    out, stats, prof = p.dev.stream_token_ids_with_stats(ids, TextGenerationConfig(10), profiled=True)
    assert out == ids + got[:10] and prof.attention > 0 and prof.mlp_projection > 0 and prof.final_logits > 0


def test_decode_stops_at_eos_and_goes_on(mixed):
    ids = mixed.ids(14, seed=10)
    cache = mixed.dev.new_kv_cache()
    mixed.dev.prefill(ids, cache)
    full, _ = mixed.dev.decode_greedy(cache, 20)
    k = next(i for i in range(3, 20) if full[i] not in full[:i])
    mixed.dev.prefill(ids, cache)
    got, _ = mixed.dev.decode_greedy(cache, 20, eos=full[k])
    assert got == full[:k] and cache.seq_len == len(ids) + k
    check(mixed.dev.forward_one(5, cache).to_host(), mixed.ref.run(ids + full[:k] + [5])[-1])


@pytest.mark.parametrize("batch", [3, 40])
def test_greedy_batch(mixed, batch):
    T, n = 9, 20
    ids = np.array([mixed.ids(T, seed=400 + b) for b in range(batch)])
    cache = mixed.dev.new_kv_cache(batch)
    want = {b: ref_greedy(mixed, [int(t) for t in ids[b]], n) for b in (0, 1, batch - 1)}
    for _ in range(3):
        mixed.dev.prefill_batch(ids, cache)
        got, _ = mixed.dev.decode_greedy_batch(cache, n)
        for b, (tokens, gaps) in want.items():
            same_until_close(got[:, b], tokens, gaps)


def test_sampled_stream(mixed):
    """A sampled stream draws what the sampler draws from the logits of single steps."""
    ids = mixed.ids(12, seed=13)
    for gen in (TextGenerationConfig(15, temperature=0.9, seed=5), TextGenerationConfig(15, temperature=1.2, top_k=7, top_p=0.9, seed=6)):
        out, _ = mixed.dev.stream_token_ids_with_stats(ids, gen)
        sampler, cache, tokens = LogitsSampler(gen.seed), mixed.dev.new_kv_cache(), list(ids)
        logits = mixed.dev.prefill(ids, cache)
        for _ in range(15):
            tokens.append(sampler.select_next_token(logits, tokens, gen))
            logits = mixed.dev.forward_one(tokens[-1], cache)
        assert out == tokens


# ---- trace runner, registry ------------------------------------------------------------------------
def test_trace_runner(mixed, tmp_path):
    a, b, c = mixed.ids(30, seed=14), mixed.ids(8, seed=15), mixed.ids(9, seed=16)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [0, 19, 7]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b, "want": [7]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[20:22], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "a", "tokens": a[22:], "want": [7]}], "end": ["a"]},
             {"step": 4, "entries": [{"id": "c", "tokens": c, "want": [0, 8]}], "end": ["c"]}]
    wa, wb, wc = mixed.ref.run(a), mixed.ref.run(b), mixed.ref.run(c)
    want = {0: wa[[0, 19, 7]], 1: wb[[7]], 3: wa[[29]], 4: wc[[0, 8]]}
    for dtype in ("bfloat16", "float32"):
        out = tmp_path / dtype
        out.mkdir()
        run_trace(mixed.dir, steps, out, dtype)
        assert sorted(os.listdir(out)) == [f"{k}.f32" for k in want]
        for k, w in want.items():
            check(np.fromfile(out / f"{k}.f32", "<f4").reshape(len(w), -1), w)


def test_registry(mixed):
    assert isinstance(mixed.dev, StackModel) and mixed.dev.architecture == "Movudra"
    assert mixed.dev.vocab_size == 61 and "architecture=Movudra" in mixed.dev.describe()
    with pytest.raises(Gpt2Error, match="weight_storage"):
        load_model(mixed.dir, Gpt2HipConfig(weight_storage=_lib.PG_STORE_INT8))
