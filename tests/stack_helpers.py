"""Stack models under test beside their oracles."""
import json
import subprocess
import sys
from pathlib import Path

import numpy as np

from puppygrad_amd import Gpt2HipConfig, _lib, load_model, synth

ROOT = Path(__file__).resolve().parents[1]
STACK_TOL = 2e-5  # root mean square difference over the vocabulary, in units of the logits' own


def rounded(w):
    """Weights as bf16 numbers."""
    return {n: synth.round_bf16(np.asarray(a, np.float32).reshape(-1)).reshape(np.shape(a)) for n, a in w.items()}


class Pair:
    """A stack model on the device and its oracle (`orc.Model`)."""

    def __init__(self, orc, tmp_path, cfg, w, storage=_lib.PG_STORE_BF16, **hip):
        synth.write_model_dir(tmp_path, cfg, w.items())
        self.dir = tmp_path
        self.dev = load_model(tmp_path, Gpt2HipConfig(weight_storage=storage, **hip))
        self.ref = orc.Model(cfg, w)
        self.vocab = cfg["vocab"]

    def ids(self, n, seed=1):
        return [int(t) for t in synth.token_ids(n, 0xA11CE + seed, self.vocab)]

    def portions(self, ids, sizes, cache=None):
        """Logits of every position, the sequence cut into portions of the given sizes (the last
        size repeats)."""
        cache = cache or self.dev.new_kv_cache()
        cache.clear()
        rows, at, k = [], 0, 0
        while at < len(ids):
            n = min(sizes[min(k, len(sizes) - 1)], len(ids) - at)
            lg = self.dev.extend(ids[at:at + n], cache, range(n)).to_host().reshape(n, -1)
            rows.append(lg)
            at, k = at + n, k + 1
        assert cache.seq_len == len(ids)
        return np.concatenate(rows)


def check(got, want, tol=STACK_TOL, what="logits"):
    got, want = np.atleast_2d(np.asarray(got, np.float64)), np.atleast_2d(want)
    assert got.shape == want.shape
    err = np.sqrt(np.mean((got - want) ** 2, axis=1)) / np.sqrt(np.mean(want ** 2))
    assert np.isfinite(got).all() and err.max() <= tol, f"{what}: {err.max():.2e} at row {err.argmax()} of {len(err)}"


def ref_greedy(p, ids, n):
    """The oracle's greedy continuation and, per step, the gap between its two best logits."""
    state, out, gaps = p.ref.new_state(), [], []
    lg = p.ref.run(ids, state)[-1]
    for _ in range(n):
        top = np.sort(lg)[-2:]
        gaps.append((top[1] - top[0]) / np.sqrt(np.mean(lg ** 2)))
        out.append(int(np.argmax(lg)))
        lg = p.ref.step(out[-1], state)
    return out, gaps


def same_until_close(got, want, gaps, tol=1e-4):
    for i, (g, w) in enumerate(zip(got, want)):
        if gaps[i] < tol:
            return i
        assert g == w, f"token {i}: {g} != {w}"
    return len(want)


def run_trace(model_dir, steps, out, dtype="bfloat16"):
    text = "".join(json.dumps(s) + "\n" for s in steps)
    r = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model", str(model_dir), "--dtype", dtype,
                        "--out", str(out), "--max-tokens", "64"], input=text, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {s['step']}" for s in steps]
