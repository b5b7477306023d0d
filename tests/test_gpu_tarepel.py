"""Tarepel on the GPU against the plain float64 oracle (oracle/tarepel.py): every mechanism alone,
prompts, portions, decoding through the cache, batches, reused caches, chunk edges, other sizes,
generation and the trace runner.  Configurations and weights are made here."""
import json
import os

import numpy as np
import pytest

import oracle.tarepel as orc
from puppygrad_amd import (Gpt2Error, Gpt2HipConfig, LogitsSampler, StackModel, TextGenerationConfig, _lib,
                           argmax_logits, generate, load_model, synth)
from stack_helpers import Pair as AnyPair, check, ref_greedy, run_trace, same_until_close

pytestmark = pytest.mark.gpu
BF16, F32 = _lib.PG_STORE_BF16, _lib.PG_STORE_F32


def attn(heads=4, kv=2, dim=16, chunk=12, rot=None, base=1000.0, scale=None):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "mask": {"size": chunk},
            "rot": {"dims": dim if rot is None else rot, "base": base},
            "scale": dim ** -0.5 if scale is None else scale}


def delta(heads=4, kv=2, dim=8, vdim=12, conv=3):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}


def parallel(left=None, right=None, ls=0.7, rs=1.3, ff=40):
    return {"type": "parallel", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"left": left or attn(), "right": right or delta(), "left_scale": ls, "right_scale": rs}}


def gla(heads=3, dim=8, vdim=20, tau=4.0, ff=24):
    return {"type": "gla", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}}


def config(layers, width=48, vocab=61, eps=1e-5, logit_scale=0.6):
    return {"architecture": "Tarepel", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "logit_scale": logit_scale, "layers": layers}


MIXED = config([parallel(), gla(), parallel(attn(6, 3, 20, 17, rot=12), delta(6, 2, 24, 16, 4), ff=None), gla(ff=None)])


def weights(cfg, seed, rank=5, **fixed):
    """Random bf16-representable weights of order-one activations; `fixed` replaces tensors (dots in
    names as __)."""
    g = np.random.default_rng(seed)
    out = {}
    for name, shape in synth.stack_tensor_shapes(cfg, rank).items():
        last = name.split(".")[-1]
        if last.startswith("norm"):
            a = 1.0 + 0.2 * g.standard_normal(shape)
        elif last in ("ls1", "ls2"):
            a = 0.5 + 0.3 * g.standard_normal(shape)
        elif last in ("pb", "dt_bias") or name.endswith("a2.b"):
            a = g.standard_normal(shape)
        elif last == "A_log":
            a = g.uniform(-2.0, 1.0, shape)
        elif last == "conv":
            a = 0.6 * g.standard_normal(shape)
        elif name == "embed":
            a = g.standard_normal(shape)
        else:
            a = g.standard_normal(shape) / np.sqrt(shape[-1])
        out[name] = synth.round_bf16(np.asarray(a, np.float32).reshape(-1)).reshape(shape)
    for name, a in fixed.items():
        name = name.replace("__", ".")
        assert out[name].shape == np.shape(a), name
        out[name] = synth.round_bf16(np.asarray(a, np.float32).reshape(-1)).reshape(np.shape(a))
    return out


class Pair(AnyPair):
    def __init__(self, *args, **kw):
        super().__init__(orc, *args, **kw)


@pytest.fixture(scope="module")
def mixed(tmp_path_factory):
    return Pair(tmp_path_factory.mktemp("mixed"), MIXED, weights(MIXED, 11))


# ---- mechanisms ------------------------------------------------------------------------------------
def zero(cfg, *names):
    shapes = synth.stack_tensor_shapes(cfg, 5)
    return {n.replace(".", "__"): np.zeros(shapes[n]) for n in names}


@pytest.mark.parametrize("left", [attn(), attn(4, 4, 16, 33, rot=6), attn(8, 1, 24, 5, base=50.0), attn(9, 1, 20, 40, rot=0),
                                  attn(20, 2, 36, 70, rot=36), attn(2, 1, 128, 300), attn(3, 3, 100, 41, rot=64), attn(2, 1, 200, 50)],
                         ids=["gqa", "mha", "mqa", "odd", "wide-group", "d128", "d100", "d200"])
def test_attention_alone(tmp_path, left):
    cfg = config([parallel(left, ff=None)])
    p = Pair(tmp_path, cfg, weights(cfg, 3, **zero(cfg, "l0.mix.right.o")))
    ids = p.ids(150)
    want = p.ref.run(ids)
    check(p.portions(ids, [len(ids)]), want, what="prompt")
    check(p.portions(ids, [1]), want, what="decoded")
    check(p.portions(ids, [50, 1, 1, 1, 7, 2, 40, 1, 2]), want, what="portions")


@pytest.mark.parametrize("right", [delta(), delta(3, 3, 16, 16, 1), delta(4, 1, 20, 40, 2), delta(2, 1, 64, 128, 4),
                                   delta(2, 2, 128, 64, 6), delta(1, 1, 4, 3, 4), delta(2, 1, 160, 200, 3), delta(1, 1, 256, 256, 4)],
                         ids=["base", "taps1", "taps2", "vdim128", "taps6", "tiny", "d160", "d256"])
def test_delta_rule_alone(tmp_path, right):
    cfg = config([parallel(right=right, ff=None)])
    p = Pair(tmp_path, cfg, weights(cfg, 4, **zero(cfg, "l0.mix.left.o")))
    ids = p.ids(75)
    want = p.ref.run(ids)
    check(p.portions(ids, [len(ids)]), want, what="prompt")
    check(p.portions(ids, [1]), want, what="decoded")
    check(p.portions(ids, [2, 3, 1, 33, 2]), want, what="portions")


@pytest.mark.parametrize("kw,rank", [(dict(), 5), (dict(heads=1, dim=32, vdim=32, tau=1.0), 1), (dict(heads=2, dim=64, vdim=128, tau=16.0), 16),
                                     (dict(heads=2, dim=100, vdim=24, tau=0.5), 20), (dict(heads=1, dim=256, vdim=256), 33),
                                     (dict(heads=5, dim=3, vdim=5), 2)], ids=["base", "tau1", "d64", "d100", "d256", "tiny"])
def test_gla_alone(tmp_path, kw, rank):
    cfg = config([gla(ff=None, **kw)])
    p = Pair(tmp_path, cfg, weights(cfg, 5, rank=rank))
    ids = p.ids(75)
    want = p.ref.run(ids)
    check(p.portions(ids, [len(ids)]), want, what="prompt")
    check(p.portions(ids, [1]), want, what="decoded")
    check(p.portions(ids, [31, 1, 2, 32, 2]), want, what="portions")


def test_strong_decays(tmp_path):
    """Decays from none to a state that is wiped by a single token, in both recurrences."""
    cfg = config([parallel(ff=None), gla(ff=None, tau=1.0)])
    w = weights(cfg, 6)
    H, n = 4, w["l1.mix.a2.b"].shape[0]
    w["l0.mix.right.A_log"] = np.linspace(-8, 4, H).astype(np.float32)
    w["l0.mix.right.a"] *= 4
    w["l1.mix.a2.b"] = synth.round_bf16(np.linspace(-60, 12, n).astype(np.float32))
    w = {k: synth.round_bf16(np.asarray(v, np.float32).reshape(-1)).reshape(np.shape(v)) for k, v in w.items()}
    p = Pair(tmp_path, cfg, w)
    ids = p.ids(140)
    want = p.ref.run(ids)
    check(p.portions(ids, [len(ids)]), want, what="prompt")
    check(p.portions(ids, [1]), want, what="decoded")


@pytest.mark.parametrize("ff", [1, 33, 200])
def test_mlp_and_norm_alone(tmp_path, ff):
    cfg = config([parallel(ff=ff)], width=37, eps=0.3, logit_scale=2.5)
    p = Pair(tmp_path, cfg, weights(cfg, 7, **zero(cfg, "l0.mix.right.o", "l0.mix.left.o")))
    ids = p.ids(40)
    want = p.ref.run(ids)
    check(p.portions(ids, [len(ids)]), want)
    check(p.portions(ids, [1]), want)


def test_extreme_scores(tmp_path):
    """Scores far into both tails of the sigmoid."""
    cfg = config([parallel(attn(4, 2, 16, 24, scale=40.0), ff=None)])
    w = weights(cfg, 8, **zero(cfg, "l0.mix.right.o"))
    p = Pair(tmp_path, cfg, w)
    ids = p.ids(60)
    want = p.ref.run(ids)
    check(p.portions(ids, [60]), want, 1e-4)  # (the scores themselves are of order 1000)
    check(p.portions(ids, [1]), want, 1e-4)


def test_many_key_splits_and_wide_sublayers(tmp_path):
    """A chunk of more key splits than the projection adds itself, and an inner width that does not
    fit beside the mixers' outputs in one launch."""
    cfg = config([parallel(attn(2, 1, 8, 700), delta(1, 1, 4, 4, 2), ff=16300)], width=16, vocab=32)
    p = Pair(tmp_path, cfg, weights(cfg, 9))
    ids = p.ids(640)
    want = p.ref.run(ids)
    check(p.portions(ids, [590, 1, 1, 1, 1, 1, 1, 1, 1, 30, 1]), want)


# ---- whole models ----------------------------------------------------------------------------------
@pytest.mark.parametrize("storage", [BF16, F32], ids=["bf16", "f32"])
@pytest.mark.parametrize("width", [48, 50, 33, 256])
def test_prompt_portions_and_decoding(tmp_path, width, storage):
    cfg = config([parallel(), gla(), parallel(attn(2, 2, 32, 19), delta(2, 1, 32, 32, 4))], width=width)
    p = Pair(tmp_path, cfg, weights(cfg, 20 + width), storage)
    ids = p.ids(101)
    want = p.ref.run(ids)
    check(p.portions(ids, [len(ids)]), want, what="prompt")
    check(p.portions(ids, [1]), want, what="decoded")
    for sizes in ([2], [3], [7], [16], [31], [32], [33], [64], [90, 1], [1, 2, 3, 5, 8, 13, 21, 34]):
        check(p.portions(ids, sizes), want, what=f"portions {sizes}")


def test_layer_order_and_first_layers(tmp_path):
    for i, layers in enumerate(([gla()], [parallel()], [gla(), gla(), parallel(ff=None)], [parallel(ff=None), gla(ff=None)])):
        cfg = config(layers)
        p = Pair(tmp_path / str(i), cfg, weights(cfg, 30 + i))
        ids = p.ids(45)
        want = p.ref.run(ids)
        check(p.portions(ids, [45]), want)
        check(p.portions(ids, [11, 1]), want)


def test_first_tokens(mixed):
    for n in (1, 2, 3, 4, 5):
        ids = mixed.ids(n, seed=40 + n)
        want = mixed.ref.run(ids)
        check(mixed.portions(ids, [n]), want, what=f"{n} tokens")
        check(mixed.portions(ids, [1]), want, what=f"{n} tokens decoded")
        cache = mixed.dev.new_kv_cache()
        check(mixed.dev.prefill(ids, cache).to_host(), want[-1])


def test_forward_matches_prefill_and_forward_one(mixed):
    ids = mixed.ids(70, seed=3)
    want = mixed.ref.run(ids)
    out = mixed.dev.forward(ids)
    check(out.logits, want)
    cache = mixed.dev.new_kv_cache()
    check(mixed.dev.prefill(ids[:-1], cache).to_host(), want[-2])
    check(mixed.dev.forward_one(ids[-1], cache).to_host(), want[-1])
    assert cache.seq_len == 70


def test_wanted_places(mixed):
    ids = mixed.ids(40, seed=4)
    want = mixed.ref.run(ids)
    cache = mixed.dev.new_kv_cache()
    assert mixed.dev.extend(ids[:20], cache, []) is None
    got = mixed.dev.extend(ids[20:], cache, [0, 3, 19])
    check(got.to_host(), want[[20, 23, 39]])
    assert [int(t) for t in got.argmax()] == [int(np.argmax(r)) for r in got.to_host()]
    for bad in ([3, 3], [4, 2], [1]):
        with pytest.raises(Gpt2Error, match="wanted places"):
            mixed.dev.extend(ids[:1], cache, bad)
    with pytest.raises(Gpt2Error, match="exceeds vocab_size"):
        mixed.dev.extend([mixed.vocab], cache)


def test_long_prompt_in_internal_segments(tmp_path):
    """More tokens than one pass over the layers takes."""
    cfg = config([parallel(attn(1, 1, 4, 50), delta(1, 1, 4, 4, 2), ff=None), gla(1, 4, 4, ff=None)], width=8, vocab=11)
    p = Pair(tmp_path, cfg, weights(cfg, 50))
    ids = p.ids(8192 + 75)
    state = p.ref.new_state()
    want = p.ref.run(ids, state)[-80:]
    cache = p.dev.new_kv_cache()
    got = p.dev.extend(ids, cache, range(len(ids) - 80, len(ids))).to_host()
    check(got, want, 1e-4)


def test_long_decoding(mixed):
    ids = mixed.ids(330, seed=5)
    want = mixed.ref.run(ids)
    check(mixed.portions(ids, [10, 1]), want)


# ---- batches, reused caches ------------------------------------------------------------------------
@pytest.mark.parametrize("batch", [2, 5, 33])
def test_batch_against_each_alone(mixed, batch):
    T, steps = 21, 16
    ids = np.array([mixed.ids(T + steps, seed=100 + b) for b in range(batch)])
    cache = mixed.dev.new_kv_cache(batch)
    got = [mixed.dev.prefill_batch(ids[:, :T], cache).to_host()]
    for t in range(T, T + steps):
        got.append(mixed.dev.forward_one_batch(ids[:, t], cache).to_host())
    got = np.stack(got, 1)
    for b in (0, 1, batch - 1):
        check(got[b], mixed.ref.run(ids[b])[T - 1:], what=f"sequence {b}")


@pytest.mark.parametrize("left,right", [(attn(4, 2, 16, 150), delta()), (attn(10, 1, 64, 90), delta(2, 1, 64, 64, 4)),
                                        (attn(2, 2, 32, 600), delta(1, 1, 128, 128, 2))], ids=["splits", "512", "1024"])
def test_batch_with_key_splits(tmp_path, left, right):
    """Blocks of every size of the one-token step, their key splits summed by a launch of their own."""
    cfg = config([parallel(left, right), parallel(left, right, ff=None)], width=64, vocab=40)
    p = Pair(tmp_path, cfg, weights(cfg, 90))
    T, steps, batch = 139, 14, 3
    ids = np.array([p.ids(T + steps, seed=500 + b) for b in range(batch)])
    cache = p.dev.new_kv_cache(batch)
    got = [p.dev.prefill_batch(ids[:, :T], cache).to_host()]
    for t in range(T, T + steps):
        got.append(p.dev.forward_one_batch(ids[:, t], cache).to_host())
    got = np.stack(got, 1)
    for b in range(batch):
        want = p.ref.run(ids[b])
        check(got[b], want[T - 1:], what=f"sequence {b}")
        check(p.portions([int(t) for t in ids[b]], [T, 1])[T - 1:], want[T - 1:], what=f"sequence {b} alone")


def test_batch_prefill_of_many_rows(mixed):
    """Enough rows for every product's tile form."""
    batch, T = 6, 90
    ids = np.array([mixed.ids(T, seed=200 + b) for b in range(batch)])
    cache = mixed.dev.new_kv_cache(batch)
    for _ in range(2):  # (the second time over what the first left)
        got = mixed.dev.prefill_batch(ids, cache).to_host()
        for b in range(batch):
            check(got[b], mixed.ref.run(ids[b])[-1])


def test_cache_used_again(mixed):
    """Sequences one after the other in one cache, in all ways to start, and rewinding."""
    cache = mixed.dev.new_kv_cache()
    long = mixed.ids(80, seed=6)
    for k, n in enumerate((33, 2, 1, 60, 5)):
        mixed.portions(long, [80], cache)
        ids = mixed.ids(n, seed=300 + k)
        want = mixed.ref.run(ids)
        check(mixed.portions(ids, [n] if k % 2 else [1], cache), want)
    with pytest.raises(Gpt2Error, match="cannot be set back"):
        cache.seq_len = 3
    cache.seq_len = 0
    check(mixed.dev.forward_one(7, cache).to_host(), mixed.ref.run([7])[-1])


def test_caches_side_by_side(mixed):
    a, b = mixed.ids(40, seed=7), mixed.ids(40, seed=8)
    wa, wb = mixed.ref.run(a), mixed.ref.run(b)
    ca, cb = mixed.dev.new_kv_cache(), mixed.dev.new_kv_cache()
    for t in range(0, 40, 4):
        check(mixed.dev.extend(a[t:t + 4], ca, range(4)).to_host(), wa[t:t + 4])
        for k in range(4):
            check(mixed.dev.forward_one(b[t + k], cb).to_host(), wb[t + k])


# ---- keys that stand out ---------------------------------------------------------------------------
def beacon_model(tmp_path, chunk, heads=2, kv=1, dim=8, far_scale=6.0, decoy=None):
    """A one-layer attention whose weights are almost 0 except for queries of token 1 on keys of
    token 2 (the last two dims of a head, which do not turn)."""
    cfg = config([parallel(attn(heads, kv, dim, chunk, rot=dim - 2, scale=1.0), ff=None)], width=32, vocab=32)
    w = weights(cfg, 60, **zero(cfg, "l0.mix.right.o"))
    C = 32
    embed = np.zeros((32, C), np.float32)
    embed[np.arange(32), np.arange(32)] = 4.0
    q, k = np.zeros((heads * dim, C), np.float32), 0.02 * np.random.default_rng(1).standard_normal((kv * dim, C))
    k[dim - 1::dim, 1:] = 0.0
    for h in range(heads):
        q[h * dim + dim - 1, 1] = far_scale
    for g in range(kv):
        k[g * dim + dim - 1, 2] = far_scale
    w["embed"], w["l0.mix.left.q"], w["l0.mix.left.k"] = embed, q, k
    w["l0.mix.left.pb"] = np.full(heads, -30.0, np.float32)
    w = {n: synth.round_bf16(np.asarray(v, np.float32).reshape(-1)).reshape(np.shape(v)) for n, v in w.items()}
    return Pair(tmp_path, cfg, w)


@pytest.mark.parametrize("chunk", [1, 2, 31, 32, 33, 64, 96, 128, 257, 300])
def test_far_key_inside_and_outside_the_chunk(tmp_path, chunk):
    p = beacon_model(tmp_path, chunk)
    start = 2 * chunk  # a chunk that does not start at 0
    fill = [3 + i % 20 for i in range(3 * chunk + 2)]
    for key, query, seen in ((start, start + chunk - 1, True), (start - 1, start, False), (start - 1, start + chunk - 1, False),
                             (start, start, False), (0, chunk - 1, True), (0, chunk, False), (start + chunk // 2, start + chunk - 1, True)):
        if key == query and seen or key >= query and key != query:
            continue
        ids = fill[:query + 1]
        ids[key] = 2
        ids[query] = 1
        if key == query:
            ids[query] = 1  # (the key is not there at all)
        seen = seen and key < query
        want = p.ref.run(ids)[-1]
        without = list(ids)
        if key < query:
            without[key] = 3
        other = p.ref.run(without)[-1]
        gap = np.sqrt(np.mean((want - other) ** 2)) / np.sqrt(np.mean(want ** 2))
        assert (gap > 0.05) == seen, (key, query, gap)  # the oracle shows whether the key is seen
        cache = p.dev.new_kv_cache()
        check(p.dev.prefill(ids, cache).to_host(), want, what=f"prompt {key} {query}")
        cache.clear()
        if query:
            p.dev.extend(ids[:-1], cache, [])
        check(p.dev.forward_one(1, cache).to_host(), want, what=f"decoded {key} {query}")
        cache.clear()
        if query >= 3:
            p.dev.extend(ids[:-2], cache, [])
            check(p.dev.extend(ids[-2:], cache).to_host(), want, what=f"two tokens {key} {query}")


def test_every_key_of_a_chunk_is_found(tmp_path):
    """One standing-out key at each place of a chunk of several splits and tiles, decoded."""
    chunk = 150
    p = beacon_model(tmp_path, chunk, heads=3, kv=1)
    cache = p.dev.new_kv_cache()
    fill = [3 + i % 20 for i in range(2 * chunk)]
    for key in list(range(0, chunk - 1, 7)) + [15, 16, 31, 32, 63, 64, 127, 128, chunk - 2]:
        ids = list(fill)
        ids[chunk + key], ids[-1] = 2, 1
        cache.clear()
        p.dev.extend(ids[:-1], cache, [])
        check(p.dev.forward_one(1, cache).to_host(), p.ref.run(ids)[-1], what=f"key {key}")


def test_old_state_in_the_first_chunks(tmp_path):
    """A write at the first token that nothing decays is still read hundreds of tokens later."""
    cfg = config([parallel(attn(1, 1, 4, 8), delta(1, 1, 8, 8, 2), ff=None), gla(1, 8, 8, ff=None)], width=24, vocab=16)
    w = weights(cfg, 70, **zero(cfg, "l0.mix.left.o"))
    w["l0.mix.right.A_log"] = np.full(1, -9.0, np.float32)
    w["l0.mix.right.b"] *= 0.1
    w["l1.mix.a2.b"] = np.full(8, 12.0, np.float32)
    p = Pair(tmp_path, cfg, {k: synth.round_bf16(np.asarray(v, np.float32).reshape(-1)).reshape(np.shape(v)) for k, v in w.items()})
    base = p.ids(400, seed=9)
    for first in (1, 2):
        ids = [first] + base[1:]
        want = p.ref.run(ids)
        check(p.portions(ids, [400]), want, 1e-4)
        check(p.portions(ids, [200, 1]), want, 1e-4)
    a, b = p.ref.run([1] + base[1:])[-1], p.ref.run([2] + base[1:])[-1]
    assert np.abs(a - b).max() > 1e-3 * np.abs(a).max()  # (the first token shows)


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
    seen = []
    out, stats = p.dev.stream_token_ids_with_stats(ids, TextGenerationConfig(25), seen.append)
    assert out == ids + got[:25] and seen == got[:25] and stats.prompt_tokens == 14
    out, stats, prof = p.dev.stream_token_ids_with_stats(ids, TextGenerationConfig(10), profiled=True)
    assert out == ids + got[:10] and prof.attention > 0 and prof.qkv_projection > 0 and prof.final_logits > 0


def test_decode_stops_at_eos_and_goes_on(mixed):
    ids = mixed.ids(14, seed=10)
    cache = mixed.dev.new_kv_cache()
    mixed.dev.prefill(ids, cache)
    full, _ = mixed.dev.decode_greedy(cache, 20)
    k = next(i for i in range(3, 20) if full[i] not in full[:i])
    mixed.dev.prefill(ids, cache)
    got, _ = mixed.dev.decode_greedy(cache, 20, eos=full[k])
    assert got == full[:k] and cache.seq_len == len(ids) + k
    # the state is that of the tokens before the EOS
    check(mixed.dev.forward_one(5, cache).to_host(), mixed.ref.run(ids + full[:k] + [5])[-1])
    out, _ = mixed.dev.stream_token_ids_with_stats(ids, TextGenerationConfig(20, eos_token_id=full[k]))
    assert out == ids + full[:k]


def test_decode_after_a_portion(mixed):
    ids = mixed.ids(30, seed=12)
    cache = mixed.dev.new_kv_cache()
    mixed.dev.extend(ids[:13], cache, [])
    with pytest.raises(Gpt2Error, match="decode needs logits"):
        mixed.dev.decode_greedy(cache, 3)
    mixed.dev.extend(ids[13:], cache, [4, 16])
    got, _ = mixed.dev.decode_greedy(cache, 10)
    want, gaps = ref_greedy(mixed, ids, 10)
    same_until_close(got, want, gaps)


def test_greedy_batch(mixed):
    batch, T, n = 3, 9, 20
    ids = np.array([mixed.ids(T, seed=400 + b) for b in range(batch)])
    cache = mixed.dev.new_kv_cache(batch)
    for _ in range(2):
        mixed.dev.prefill_batch(ids, cache)
        got, _ = mixed.dev.decode_greedy_batch(cache, n)
        for b in range(batch):
            want, gaps = ref_greedy(mixed, [int(t) for t in ids[b]], n)
            same_until_close(got[:, b], want, gaps)


def test_sampled_stream(mixed):
    """A sampled stream draws what the sampler draws from the logits of single steps."""
    ids = mixed.ids(12, seed=13)
    for gen in (TextGenerationConfig(15, temperature=0.9, seed=5), TextGenerationConfig(15, temperature=1.2, top_k=7, top_p=0.9, seed=6),
                TextGenerationConfig(15, repeat_penalty=1.5, repeat_last_n=6)):
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
             {"step": 1, "entries": [{"id": "b", "tokens": b, "want": [7]}, {"id": "a", "tokens": a[20:22], "want": []}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[22:23], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "a", "tokens": a[23:], "want": [6]}, {"id": "c", "tokens": c, "want": [0, 8]}], "end": ["a", "c"]}]
    wa, wb, wc = mixed.ref.run(a), mixed.ref.run(b), mixed.ref.run(c)
    want = {0: wa[[0, 19, 7]], 1: wb[[7]], 3: np.concatenate([wa[[29]], wc[[0, 8]]])}
    for dtype in ("bfloat16", "float32"):
        out = tmp_path / dtype
        out.mkdir()
        run_trace(mixed.dir, steps, out, dtype)
        assert sorted(os.listdir(out)) == ["0.f32", "1.f32", "3.f32"]
        for k, w in want.items():
            check(np.fromfile(out / f"{k}.f32", "<f4").reshape(len(w), -1), w)


def test_registry_and_gpt2_portions(tmp_path, mixed):
    """The registry tells the architectures apart; a GPT-2 takes portions too."""
    from puppygrad_amd import Gpt2Config, Gpt2Model
    from test_assets import write_model_dir
    assert isinstance(mixed.dev, StackModel) and mixed.dev.architecture == "Tarepel"
    assert mixed.dev.vocab_size == 61 and "architecture=Tarepel" in mixed.dev.describe()
    cfg = Gpt2Config(vocab_size=131, n_positions=40, n_embd=128, n_layer=2, n_head=2)
    write_model_dir(tmp_path, cfg, synth.random_weights(cfg, 0x5EED0901, perturb=True))
    model = load_model(tmp_path)
    assert isinstance(model, Gpt2Model) and model.architecture == "gpt2"
    ids = [int(t) for t in synth.token_ids(17, 3, 131)]
    want = model.forward(ids).logits
    for sizes in ([17], [5, 1, 11], [1]):
        cache, at = model.new_kv_cache(), 0
        for n in sizes * 17:
            n = min(n, len(ids) - at)
            if n == 0:
                break
            got = model.extend(ids[at:at + n], cache, range(n)).to_host().reshape(n, -1)
            np.testing.assert_allclose(got, want[at:at + n], atol=1e-4, rtol=1e-3)
            at += n
    with pytest.raises(Gpt2Error, match="made for another model"):
        mixed.dev.prefill([1, 2], model.new_kv_cache())
    with pytest.raises(Gpt2Error, match="weight_storage"):
        load_model(mixed.dir, Gpt2HipConfig(weight_storage=_lib.PG_STORE_INT8))


def test_float32_checkpoint_and_argmax(tmp_path):
    """F32 tensors load too, and are rounded to bf16 only for bf16 storage."""
    cfg = config([parallel(), gla()])
    w = weights(cfg, 80)
    w["l0.mix.left.q"] = w["l0.mix.left.q"] * np.float32(1.0 + 2 ** -12)  # not a bf16 number
    synth.write_model_dir(tmp_path, cfg, w.items())
    header, at, body = {}, 0, b""
    for name, a in w.items():
        raw = np.ascontiguousarray(a, np.float32).tobytes()
        header[name] = {"dtype": "F32", "shape": list(a.shape), "data_offsets": [at, at + len(raw)]}
        at += len(raw)
        body += raw
    text = json.dumps(header).encode()
    (tmp_path / "model.safetensors").write_bytes(len(text).to_bytes(8, "little") + text + body)
    ids = [int(t) for t in synth.token_ids(30, 5, 61)]
    exact = orc.Model(cfg, w).run(ids)
    rounded = orc.Model(cfg, {k: synth.round_bf16(np.asarray(v, np.float32).reshape(-1)).reshape(v.shape) for k, v in w.items()}).run(ids)
    got = load_model(tmp_path, Gpt2HipConfig(weight_storage=F32)).forward(ids).logits
    check(got, exact)
    check(load_model(tmp_path, Gpt2HipConfig(weight_storage=BF16)).forward(ids).logits, rounded)
    assert argmax_logits(got[-1]) == int(np.argmax(got[-1]))
