"""TEST INFRASTRUCTURE ONLY: a plain, slow Movudra in float64, one function per mechanism.

Everything runs one token (and one head) at a time, straight from the equations, and shares
no code with the product path.  `Model` keeps the per-sequence state in ordinary Python
lists, so that a whole prompt, portions of it and single tokens all run the same loop.

Notation: h is a sublayer's input vector, W_x the matrix `<layer>.mix.x` ([out, in], applied as
W x); `sigmoid`, `silu(z) = z sigmoid(z)`.
"""
from __future__ import annotations

import math

import numpy as np

from .tarepel import delta_decay, rms, short_conv, sigmoid, silu, softplus, unit


# ---- rotation ----------------------------------------------------------------------------------
def yarn_frequencies(dims, base, scaling):
    """Angles per position of the dims / 2 pairs, and the factor of sine and cosine: between the
    pairs that turn `fast` and `slow` times over `original` positions the frequencies go over
    from f to f / factor."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return f, 1.0

    def pair_of(turns):
        return dims * math.log(scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_of(scaling["fast"])), 0)
    hi = min(math.ceil(pair_of(scaling["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / scaling["factor"] * r + fi * (1.0 - r))
    return out, 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_pairs(x, pos, freqs, mag):
    """The pairs (2 i, 2 i + 1) turn by pos * freqs[i] and grow by mag; the rest passes."""
    y = x.copy()
    for i, f in enumerate(freqs):
        c, s = mag * math.cos(pos * f), mag * math.sin(pos * f)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i] = u * c - v * s
        y[..., 2 * i + 1] = v * c + u * s
    return y


# ---- attention ---------------------------------------------------------------------------------
def window_start(pos, size):
    """First position that position `pos` sees."""
    return max(0, pos - size + 1)


def sink_attention(q, keys, values, scale, sink):
    """One head: q [d] against keys [n][d], values [n][e]; softmax whose denominator also holds
    exp(sink)."""
    z = keys @ q * scale
    m = max(float(np.max(z)), float(sink))
    w = np.exp(z - m)
    return (w / (np.sum(w) + math.exp(sink - m))) @ values


# ---- recurrences ---------------------------------------------------------------------------------
def ssd_step(S, a, dt, B, C, x):
    """One head of a state-space step: S [N][vdim] decays by exp(a dt), takes dt B x^T, is read at C."""
    S = math.exp(a * dt) * S + dt * np.outer(B, x)
    return S, S.T @ C


def channel_delta_step(S, q, k, v, g, beta):
    """One head's delta rule with a decay g per key channel: S [dim][vdim]; decay, write, read."""
    S = g[:, None] * S
    u = beta * (v - S.T @ k)
    S = S + np.outer(k, u)
    return S, S.T @ q


def group_rms(y, groups, eps):
    return rms(y.reshape(groups, -1), eps).reshape(-1)


# ---- feed-forward --------------------------------------------------------------------------------
def softmax(z):
    e = np.exp(z - np.max(z))
    return e / np.sum(e)


def route(z, top):
    """The chosen experts (largest scores first) and their weights: softmax over all experts."""
    s = softmax(z)
    order = np.argsort(-s, kind="stable")[:top]
    return order, s[order]


# ---- the model -------------------------------------------------------------------------------------
class State:
    """What one sequence carries from token to token."""

    def __init__(self, cfg):
        self.pos = 0
        self.layers = []
        for layer in cfg["layers"]:
            m, t = layer["mixer"], layer["type"]
            if t == "mamba2":
                ch = m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]
                self.layers.append({"S": np.zeros((m["heads"], m["state"], m["vdim"])),
                                    "conv": [np.zeros(ch)] * (m["conv"] - 1)})
            elif t == "channel_delta":
                n = {"q": m["kv_heads"] * m["dim"], "k": m["kv_heads"] * m["dim"], "v": m["heads"] * m["vdim"]}
                self.layers.append({"S": np.zeros((m["heads"], m["dim"], m["vdim"])),
                                    **{x: [np.zeros(c)] * (m["conv"] - 1) for x, c in n.items()}})
            else:
                self.layers.append({"c": [], "r": []})


class Model:
    def __init__(self, cfg, tensors):
        self.cfg = cfg
        self.w = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
        self.eps = cfg["norm"]["eps"]

    def new_state(self):
        return State(self.cfg)

    def mamba2(self, p, c, h, st):
        w = self.w
        H, e, N, G = c["heads"], c["vdim"], c["state"], c["groups"]
        inner = H * e
        z, xbc, dt = np.split(w[p + "in"] @ h, [inner, 2 * inner + 2 * G * N])
        window = st["conv"] + [xbc]
        st["conv"] = window[1:]
        taps = w[p + "conv"]
        s = np.sum(np.stack(window) * taps.T, axis=0) + w[p + "conv.b"]
        x, B, C = np.split(silu(s), [inner, inner + G * N])
        x, B, C = x.reshape(H, e), B.reshape(G, N), C.reshape(G, N)
        dt = softplus(dt + w[p + "dt_bias"])
        y = np.zeros((H, e))
        for i in range(H):
            g = i // (H // G)
            st["S"][i], o = ssd_step(st["S"][i], -math.exp(w[p + "A_log"][i]), dt[i], B[g], C[g], x[i])
            y[i] = o + w[p + "D"][i] * x[i]
        y = group_rms(y.reshape(-1) * silu(z), c["norm_groups"], self.eps) * w[p + "norm"]
        return w[p + "o"] @ y

    def channel_delta(self, p, c, h, st):
        w = self.w
        H, G, d, e = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
        x = {}
        for name in ("q", "k", "v"):
            window = st[name] + [w[p + name] @ h]
            x[name] = short_conv(np.stack(window), w[p + name + ".conv"])
            st[name] = window[1:]
        q = unit(x["q"].reshape(G, d)) * d ** -0.5
        k = unit(x["k"].reshape(G, d))
        v = x["v"].reshape(H, e)
        beta = sigmoid(w[p + "b"] @ h)
        a = (w[p + "a2"] @ (w[p + "a1"] @ h)).reshape(H, d)
        g = delta_decay(a, w[p + "A_log"][:, None], w[p + "dt_bias"].reshape(H, d))
        o = np.zeros((H, e))
        for i in range(H):
            j = i // (H // G)
            st["S"][i], o[i] = channel_delta_step(st["S"][i], q[j], k[j], v[i], g[i], beta[i])
        gate = sigmoid(w[p + "g2"] @ (w[p + "g1"] @ h)).reshape(H, e)
        return w[p + "o"] @ (rms(o, self.eps) * w[p + "norm"] * gate).reshape(-1)

    def latent_attention(self, p, c, h, st, pos):
        w = self.w
        H, d, r, e, K = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
        rot = c["rot"]
        freqs, mag = yarn_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
        q = (w[p + "uq"] @ (rms(w[p + "dq"] @ h, self.eps) * w[p + "dq.norm"])).reshape(H, d + r)
        kv = w[p + "dkv"] @ h
        st["c"].append(rms(kv[:K], self.eps) * w[p + "dkv.norm"])
        st["r"].append(rotate_pairs(kv[K:], pos, freqs, mag))
        lo = window_start(pos, c["mask"]["size"])
        lat, rk = np.stack(st["c"][lo:pos + 1]), np.stack(st["r"][lo:pos + 1])
        uk, uv = w[p + "uk"].reshape(H, d, K), w[p + "uv"].reshape(H, e, K)
        o = np.zeros((H, e))
        for i in range(H):
            qi = np.concatenate([q[i, :d], rotate_pairs(q[i, d:], pos, freqs, mag)])
            keys = np.concatenate([lat @ uk[i].T, rk], axis=1)
            o[i] = sink_attention(qi, keys, lat @ uv[i].T, c["scale"], w[p + "sink"][i])
        return w[p + "o"] @ o.reshape(-1)

    def dense(self, p, h):
        w = self.w
        a = np.maximum(w[p + "up"] @ h + w[p + "up.b"], 0.0) ** 2
        return w[p + "down"] @ a + w[p + "down.b"]

    def moe(self, p, c, h):
        w = self.w
        chosen, weights = route(w[p + "router"] @ h, c["router"]["top"])
        out = np.zeros_like(h)
        for i, s in zip(chosen, weights):
            e = f"{p}e{i}."
            out += s * (w[e + "down"] @ (silu(w[e + "gate"] @ h) * (w[e + "up"] @ h)))
        return out

    def norm(self, x, name):
        return rms(x, self.eps) * self.w[name]

    def layer(self, i, x, st, pos):
        c = self.cfg["layers"][i]
        p, m = f"l{i}.mix.", c["mixer"]
        if c["type"] == "mamba2":
            mix = self.mamba2(p, m, x, st)
        elif c["type"] == "channel_delta":
            mix = self.channel_delta(p, m, x, st)
        else:
            mix = self.latent_attention(p, m, x, st, pos)
        x = x + self.norm(mix, f"l{i}.norm1")
        f = c.get("mlp")
        if f:
            y = self.dense(f"l{i}.mlp.", x) if f["kind"] == "dense" else self.moe(f"l{i}.mlp.", f, x)
            x = x + self.norm(y, f"l{i}.norm2")
        return x

    def step(self, token, state, residuals=None):
        x = self.w["embed"][token].copy()
        for i in range(len(self.cfg["layers"])):
            x = self.layer(i, x, state.layers[i], state.pos)
            if residuals is not None:
                residuals[i].append(x)
        state.pos += 1
        return self.w["head"] @ self.norm(x, "final.norm")

    def run(self, tokens, state=None, residuals=None):
        """Logits at every position of `tokens`, continuing from `state`."""
        state = state or self.new_state()
        return np.stack([self.step(int(t), state, residuals) for t in tokens])
