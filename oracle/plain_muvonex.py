"""Muvonex in plain numpy: one function per mechanism, one token at a time, recurrences as they are written.

Independent of the product: no code, table or layout is shared with it.  Everything runs in float64; weights come in as a
dict name -> array (any float type), the configuration as the parsed config.json.

    run(cfg, w, tokens)            -> Trace(logits [T, vocab], layers [layers, T, width])
    Sequence(cfg, w).step(tokens)  -> the same logits, portion by portion, from what earlier tokens left behind
"""
from __future__ import annotations

from collections import namedtuple

import numpy as np

Trace = namedtuple("Trace", "logits layers")


def rms(x, eps):
    """x over its root mean square along the last axis, eps under the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def zero_centred_norm(x, weight, eps):
    """RMS norm whose weight is stored as its distance from one."""
    return rms(x, eps) * (1.0 + weight)


def silu(z):
    return z / (1.0 + np.exp(-z))


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def unit(x):
    """Unit vector along the last axis; 1e-6 under the root keeps a zero vector finite."""
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def frequency(i, rot):
    """Turning rate of rotated pair i: base^(-2i/dims); slow pairs are slowed further by `factor`, those in between blended."""
    f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
    s = rot.get("scaling")
    if not s:
        return f
    length = 2.0 * np.pi / f
    if length < s["original"] / s["high"]:
        return f
    if length > s["original"] / s["low"]:
        return f / s["factor"]
    t = (s["original"] / length - s["low"]) / (s["high"] - s["low"])
    return (1.0 - t) * f / s["factor"] + t * f


def rotate_half(v, position, rot):
    """Rotary embedding along the last axis: element i < dims/2 turns with element i + dims/2, elements from dims on stay."""
    out = np.array(v, copy=True)
    half = rot["dims"] // 2
    for i in range(half):
        a = position * frequency(i, rot)
        c, s = np.cos(a), np.sin(a)
        out[..., i] = v[..., i] * c - v[..., i + half] * s
        out[..., i + half] = v[..., i + half] * c + v[..., i] * s
    return out


def softmax_with_sink(scores, sink):
    """Weights of the keys; exp(sink) joins the denominator and nothing else."""
    m = max(float(np.max(scores)), float(sink))
    e = np.exp(scores - m)
    return e / (np.sum(e) + np.exp(sink - m))


def short_conv(window, weight, bias=0.0):
    """window [taps, channels], oldest first, the current token last."""
    return np.sum(window * weight.T, axis=0) + bias


class Window:
    """The last taps - 1 inputs of a short convolution; zeros before the start."""

    def __init__(self, taps, channels):
        self.past = np.zeros((taps - 1, channels))

    def push(self, x):
        w = np.concatenate([self.past, x[None]])
        self.past = w[1:]
        return w


def grouped_attention(h, position, history, mix, p, w, eps):
    """One token through softmax attention with shared key/value heads and a sink per head; history: (k, v) per position."""
    nh, ng, dim, vdim = mix["heads"], mix["kv_heads"], mix["dim"], mix["vdim"]
    q = rms(rotate_half((w[p + "q"] @ h).reshape(nh, dim), position, mix["rot"]), eps)
    k = rms(rotate_half((w[p + "k"] @ h).reshape(ng, dim), position, mix["rot"]), eps)
    history.append((k, (w[p + "v"] @ h).reshape(ng, vdim)))
    keys, vals = np.stack([a for a, _ in history]), np.stack([b for _, b in history])
    outs = []
    for j in range(nh):
        g = j // (nh // ng)
        outs.append(softmax_with_sink(keys[:, g] @ q[j] * mix["scale"], float(w[p + "sink"][j])) @ vals[:, g])
    return w[p + "o"] @ np.concatenate(outs)


def ssd_update(state, decay, dt, x, b, c, skip):
    """One head, one token of the diagonal-decay state space: state [N, vdim] -> (state, output)."""
    state = decay * state + dt * np.outer(b, x)
    return state, state.T @ c + skip * x


def state_space(h, memory, mix, p, w, eps):
    nh, vd, n, ng, parts = mix["heads"], mix["vdim"], mix["state"], mix["groups"], mix["norm_groups"]
    inner = nh * vd
    z, xbc, dt = np.split(w[p + "in"] @ h, [inner, 2 * inner + 2 * ng * n])
    if memory.get("conv") is None:
        memory["conv"] = Window(mix["conv"], inner + 2 * ng * n)
        memory["s"] = np.zeros((nh, n, vd))
    xbc = silu(short_conv(memory["conv"].push(xbc), w[p + "conv"], w[p + "conv.b"]))
    x, b, c = np.split(xbc, [inner, inner + ng * n])
    x, b, c = x.reshape(nh, vd), b.reshape(ng, n), c.reshape(ng, n)
    dt = softplus(dt + w[p + "dt_bias"])
    y = np.zeros((nh, vd))
    for j in range(nh):
        g = j // (nh // ng)
        decay = np.exp(-np.exp(w[p + "A_log"][j]) * dt[j])
        memory["s"][j], y[j] = ssd_update(memory["s"][j], decay, dt[j], x[j], b[g], c[g], w[p + "D"][j])
    y = (y.reshape(inner) * silu(z)).reshape(parts, inner // parts)
    return w[p + "o"] @ (rms(y, eps).reshape(inner) * w[p + "norm"])


def delta_update(state, decay, beta, q, k, v):
    """One head, one token of the gated delta rule: state [dim, vdim] -> (state, output)."""
    state = decay * state
    u = beta * (v - state.T @ k)
    state = state + np.outer(k, u)
    return state, state.T @ q


def gated_delta(h, memory, mix, p, w, eps):
    nh, nk, dim, vd = mix["heads"], mix["kv_heads"], mix["dim"], mix["vdim"]
    if memory.get("s") is None:
        memory["s"] = np.zeros((nh, dim, vd))
        for t, n in (("q", nk * dim), ("k", nk * dim), ("v", nh * vd)):
            memory[t] = Window(mix["conv"], n)
    q, k, v = (silu(short_conv(memory[t].push(w[p + t] @ h), w[p + t + ".conv"])) for t in "qkv")
    q = unit(q.reshape(nk, dim)) * dim ** -0.5
    k = unit(k.reshape(nk, dim))
    v = v.reshape(nh, vd)
    beta = sigmoid(w[p + "b"] @ h)
    decay = np.exp(-np.exp(w[p + "A_log"]) * softplus(w[p + "a"] @ h + w[p + "dt_bias"]))
    o = np.zeros((nh, vd))
    for j in range(nh):
        g = j // (nh // nk)
        memory["s"][j], o[j] = delta_update(memory["s"][j], decay[j], beta[j], q[g], k[g], v[j])
    o = rms(o, eps) * w[p + "norm"] * silu((w[p + "g"] @ h).reshape(nh, vd))
    return w[p + "o"] @ o.reshape(-1)


def mixer(h, position, memory, layer, p, w, eps):
    mix = layer["mixer"]
    if layer["type"] == "delta":
        return gated_delta(h, memory, mix, p, w, eps)
    left = grouped_attention(h, position, memory.setdefault("kv", []), mix["left"], p + "left.", w, eps)
    right = state_space(h, memory, mix["right"], p + "right.", w, eps)
    return mix["left_scale"] * left + mix["right_scale"] * right


def gated_mlp(h, p, w):
    return w[p + "down"] @ (gelu_tanh(w[p + "gate"] @ h) * (w[p + "up"] @ h))


class Sequence:
    """One request: per layer the keys and values so far, the recurrent states and the short convolutions' windows."""

    def __init__(self, cfg, w):
        self.cfg = cfg
        self.w = {k: np.asarray(v, dtype=np.float64) for k, v in w.items()}
        self.memory = [{} for _ in cfg["layers"]]
        self.position = 0

    def token(self, tok):
        """-> (logits, residual stream after every layer)"""
        cfg, w, eps = self.cfg, self.w, self.cfg["norm"]["eps"]
        x, states = w["embed"][int(tok)] * cfg["embedding"]["scale"], []
        for i, layer in enumerate(cfg["layers"]):
            p = f"l{i}."
            h = zero_centred_norm(x, w[p + "norm1"], eps)
            y = mixer(h, self.position, self.memory[i], layer, p + "mix.", w, eps)
            if layer.get("mlp"):
                y = y + gated_mlp(h, p + "mlp.", w)
            x = x + cfg["residual_mult"] * y
            states.append(x)
        self.position += 1
        return w["embed"] @ zero_centred_norm(x, w["final.norm"], eps), np.stack(states)

    def step(self, tokens):
        return np.stack([self.token(t)[0] for t in tokens])


def run(cfg, w, tokens):
    s = Sequence(cfg, w)
    rows = [s.token(t) for t in tokens]
    return Trace(np.stack([a for a, _ in rows]), np.stack([b for _, b in rows], axis=1))
