"""TEST INFRASTRUCTURE ONLY: a plain, slow Tarepel in float64, one function per mechanism.

Everything runs one token (and one head) at a time, straight from the equations, and shares
no code with the product path.  `Model` keeps the per-sequence state in ordinary Python
lists, so that a whole prompt, portions of it and single tokens all run the same loop.

Notation: h is a mixer's input vector, W_x the matrix `<layer>.mix.x` ([out, in], applied as
W x); `sigmoid`, `silu(z) = z sigmoid(z)`.
"""
from __future__ import annotations

import math

import numpy as np


# ---- scalar and vector functions -------------------------------------------------------------
def sigmoid(z):
    z = np.asarray(z, np.float64)
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rms(x, eps):
    """x over its root mean square along the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def unit(x):
    """x as a unit vector along the last axis."""
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def rotate(x, pos, dims, base):
    """Rotary positions on the first `dims` values: the pair (i, i + dims/2) turns by
    pos * base^(-2 i / dims)."""
    y = x.copy()
    half = dims // 2
    for i in range(half):
        a = pos * base ** (-2.0 * i / dims)
        c, s = math.cos(a), math.sin(a)
        u, v = x[..., i], x[..., i + half]
        y[..., i] = u * c - v * s
        y[..., i + half] = v * c + u * s
    return y


# ---- mechanisms ----------------------------------------------------------------------------------
def chunk_start(pos, size):
    """First position that shares a chunk with `pos`."""
    return pos // size * size


def sigmoid_attention(q, keys, values, scale, head_bias, groups):
    """q [H][d] against keys [n][G][d] and values [n][G][e]: every key weighs
    sigmoid(q . k * scale + bias of the head), without normalisation."""
    H = q.shape[0]
    out = np.zeros((H, values.shape[-1]))
    for h in range(H):
        g = h // (H // groups)
        w = sigmoid(keys[:, g] @ q[h] * scale + head_bias[h])
        out[h] = w @ values[:, g]
    return out


def short_conv(window, taps):
    """window [taps][channels] (the last row is the current token's), taps [channels][taps]."""
    return silu(np.sum(window * taps.T, axis=0))


def delta_step(S, q, k, v, g, beta):
    """One head's gated delta rule: S [dim][vdim]; decay, write, then read at q."""
    S = g * S
    u = beta * (v - S.T @ k)
    S = S + np.outer(k, u)
    return S, S.T @ q


def gla_step(S, q, k, v, alpha):
    """One head's linear attention with a decay per key channel: S [dim][vdim]."""
    S = alpha[:, None] * S + np.outer(k, v)
    return S, S.T @ q


def delta_decay(a, A_log, dt_bias):
    return np.exp(-np.exp(A_log) * softplus(a + dt_bias))


def gla_decay(z, tau):
    return sigmoid(z) ** (1.0 / tau)


# ---- the model -------------------------------------------------------------------------------------
class State:
    """What one sequence carries from token to token."""

    def __init__(self, cfg):
        self.pos = 0
        self.layers = []
        for layer in cfg["layers"]:
            m = layer["mixer"]
            if layer["type"] == "parallel":
                R = m["right"]
                taps = R["conv"]
                self.layers.append({
                    "keys": [], "values": [],
                    "S": np.zeros((R["heads"], R["dim"], R["vdim"])),
                    "q": [np.zeros(R["kv_heads"] * R["dim"])] * (taps - 1),
                    "k": [np.zeros(R["kv_heads"] * R["dim"])] * (taps - 1),
                    "v": [np.zeros(R["heads"] * R["vdim"])] * (taps - 1)})
            else:
                self.layers.append({"S": np.zeros((m["heads"], m["dim"], m["vdim"]))})


class Model:
    def __init__(self, cfg, tensors):
        self.cfg = cfg
        self.w = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
        self.eps = cfg["norm"]["eps"]

    def new_state(self):
        return State(self.cfg)

    def left(self, p, c, h, st, pos):
        w = self.w
        H, G, d = c["heads"], c["kv_heads"], c["dim"]
        rot = c["rot"]
        q = (w[p + "q"] @ h).reshape(H, d)
        k = (w[p + "k"] @ h).reshape(G, d)
        st["keys"].append(rotate(k, pos, rot["dims"], rot["base"]))
        st["values"].append(k)
        lo = chunk_start(pos, c["mask"]["size"])
        keys, values = np.stack(st["keys"][lo:pos + 1]), np.stack(st["values"][lo:pos + 1])
        o = sigmoid_attention(rotate(q, pos, rot["dims"], rot["base"]), keys, values, c["scale"],
                              w[p + "pb"], G)
        return w[p + "o"] @ o.reshape(-1)

    def right(self, p, c, h, st):
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
        g = delta_decay(w[p + "a"] @ h, w[p + "A_log"], w[p + "dt_bias"])
        o = np.zeros((H, e))
        for i in range(H):
            j = i // (H // G)
            st["S"][i], o[i] = delta_step(st["S"][i], q[j], k[j], v[i], g[i], beta[i])
        y = rms(o, self.eps) * w[p + "norm"] * silu(w[p + "g"] @ h).reshape(H, e)
        return w[p + "o"] @ y.reshape(-1)

    def gla(self, p, c, h, st):
        w = self.w
        H, d, e = c["heads"], c["dim"], c["vdim"]
        q = (w[p + "q"] @ h).reshape(H, d) * d ** -0.5
        k = (w[p + "k"] @ h).reshape(H, d)
        v = (w[p + "v"] @ h).reshape(H, e)
        z = w[p + "a2"] @ (w[p + "a1"] @ h) + w[p + "a2.b"]
        alpha = gla_decay(z, c["tau"]).reshape(H, d)
        o = np.zeros((H, e))
        for i in range(H):
            st["S"][i], o[i] = gla_step(st["S"][i], q[i], k[i], v[i], alpha[i])
        y = (rms(o, self.eps) * w[p + "norm"]).reshape(-1) * silu(w[p + "g"] @ h)
        return w[p + "o"] @ y

    def mlp(self, p, h):
        w = self.w
        return w[p + "down"] @ (gelu_tanh(w[p + "gate"] @ h) * (w[p + "up"] @ h))

    def layer(self, i, x, st, pos):
        c, w = self.cfg["layers"][i], self.w
        h = rms(x, self.eps) * w[f"l{i}.norm1"]
        p, m = f"l{i}.mix.", c["mixer"]
        if c["type"] == "parallel":
            mix = (m["left_scale"] * self.left(p + "left.", m["left"], h, st, pos)
                   + m["right_scale"] * self.right(p + "right.", m["right"], h, st))
        else:
            mix = self.gla(p, m, h, st)
        y = x + w[f"l{i}.ls1"] * mix
        if c.get("mlp"):
            y = y + w[f"l{i}.ls2"] * self.mlp(f"l{i}.mlp.", h)
        return y

    def step(self, token, state, residuals=None):
        x = self.w["embed"][token].copy()
        for i in range(len(self.cfg["layers"])):
            x = self.layer(i, x, state.layers[i], state.pos)
            if residuals is not None:
                residuals[i].append(x)
        state.pos += 1
        return self.w["head"] @ (rms(x, self.eps) * self.w["final.norm"]) * self.cfg["logit_scale"]

    def run(self, tokens, state=None, residuals=None):
        """Logits at every position of `tokens`, continuing from `state`."""
        state = state or self.new_state()
        return np.stack([self.step(int(t), state, residuals) for t in tokens])
