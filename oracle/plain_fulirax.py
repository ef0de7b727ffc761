"""Fulirax in plain numpy: one function per mechanism, one token and one head at a time where that is the clearest form.

Independent of the product: no code, table or layout is shared with it.  Everything runs in float64 unless a dtype is
given; weights come in as a dict name -> array (any float type), the configuration as the parsed config.json.

    run_prompt(cfg, w, tokens)     -> logits [T, vocab] of a whole prompt in matrix form
    run(cfg, w, tokens)            -> Trace(logits [T, vocab], layers [runs, T, width])
    Sequence(cfg, w).step(tokens)  -> the same logits, portion by portion, from a per-pass history of latents
"""
from __future__ import annotations

from collections import namedtuple

import numpy as np

Trace = namedtuple("Trace", "logits layers")


def dynamic_tanh(x, alpha, weight, bias):
    """tanh(alpha x) * weight + bias, elementwise: no statistics of the row enter."""
    return np.tanh(alpha * x) * weight + bias


def rms_norm(x, weight, eps):
    """x over its root mean square (eps under the root), times weight."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * weight


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def rotate_half(v, position, base, dims):
    """Rotary embedding of one vector: element i < dims/2 turns with element i + dims/2, elements from dims on stay."""
    out = np.array(v, copy=True)
    half = dims // 2
    for i in range(half):
        a = position * float(base) ** (-2.0 * i / dims)
        c, s = np.cos(a), np.sin(a)
        out[i] = v[i] * c - v[i + half] * s
        out[i + half] = v[i + half] * c + v[i] * s
    return out


def softmax_with_sink(scores, sink):
    """Weights of the keys; exp(sink) joins the denominator and nothing else."""
    m = max(float(np.max(scores)), float(sink))
    e = np.exp(scores - m)
    return e / (np.sum(e) + np.exp(sink - m))


def latent_entry(h, position, mix, p, w, eps):
    """What one token leaves behind for later tokens: the normed latent and the one rotated key part of all heads."""
    kv = w[p + "dkv"] @ h
    c = rms_norm(kv[: mix["kv_rank"]], w[p + "dkv.norm"], eps)
    return c, rotate_half(kv[mix["kv_rank"]:], position, mix["rot"]["base"], mix["rot"]["dims"])


def latent_attention(h, position, history, mix, p, w):
    """One query token over `history`, the list of (latent, rotated key part) of positions 0 .. its own."""
    nh, dim, rot, vdim = mix["heads"], mix["dim"], mix["rot_dim"], mix["vdim"]
    q = (w[p + "q"] @ h).reshape(nh, dim + rot)
    lat = np.stack([c for c, _ in history])
    kr = np.stack([r for _, r in history])
    outs = []
    for j in range(nh):
        k = lat @ w[p + "uk"][j * dim:(j + 1) * dim].T
        v = lat @ w[p + "uv"][j * vdim:(j + 1) * vdim].T
        qr = rotate_half(q[j, dim:], position, mix["rot"]["base"], mix["rot"]["dims"])
        s = (k @ q[j, :dim] + kr @ qr) * mix["scale"]
        outs.append(softmax_with_sink(s, float(w[p + "sink"][j])) @ v)
    return w[p + "o"] @ np.concatenate(outs)


def dense_mlp(h, p, w):
    return w[p + "down"] @ gelu_tanh(w[p + "up"] @ h)


def norm(x, name, w):
    return dynamic_tanh(x, float(np.asarray(w[name + ".alpha"]).reshape(())), w[name], w[name + ".b"])


def loop_entry(x, x0, t, w):
    """Start of pass t of the repeated layers: mix the stream with the embedding output, add the pass's vector."""
    return w["loop.in"] @ np.concatenate([x, x0]) + w["loop.step"][t]


def schedule(cfg):
    """Layer runs in order: (layer, pass or None, True on the first layer of a pass)."""
    n, loop, out, i = len(cfg["layers"]), cfg.get("loop"), [], 0
    while i < n:
        if loop and i == loop["start"]:
            for t in range(loop["times"]):
                out += [(L, t, L == loop["start"]) for L in range(loop["start"], loop["stop"])]
            i = loop["stop"]
        else:
            out.append((i, None, False))
            i += 1
    return out


class Sequence:
    """One request: a history of (latent, rotated key part) per layer run."""

    def __init__(self, cfg, w):
        self.cfg = cfg
        self.w = {k: np.asarray(v, dtype=np.float64) for k, v in w.items()}
        self.runs = schedule(cfg)
        self.history = [[] for _ in self.runs]
        self.position = 0

    def token(self, tok):
        """-> (logits, residual stream after every layer run)"""
        cfg, w, eps = self.cfg, self.w, self.cfg["norm"]["eps"]
        x0 = w["embed"][int(tok)]
        x, states = x0, []
        for r, (L, t, first) in enumerate(self.runs):
            if first:
                x = loop_entry(x, x0, t, w)
            p, layer = f"l{L}.", cfg["layers"][L]
            h = norm(x, p + "norm1", w)
            self.history[r].append(latent_entry(h, self.position, layer["mixer"], p + "mix.", w, eps))
            x = x + latent_attention(h, self.position, self.history[r], layer["mixer"], p + "mix.", w)
            if layer.get("mlp"):
                x = x + dense_mlp(norm(x, p + "norm2", w), p + "mlp.", w)
            states.append(x)
        self.position += 1
        return w["embed"] @ norm(x, "final.norm", w) * cfg["logit_scale"], np.stack(states)

    def step(self, tokens):
        return np.stack([self.token(t)[0] for t in tokens])


def run(cfg, w, tokens):
    s = Sequence(cfg, w)
    rows = [s.token(t) for t in tokens]
    return Trace(np.stack([a for a, _ in rows]), np.stack([b for _, b in rows], axis=1))


def run_prompt(cfg, w, tokens):
    """The same equations for all positions of one prompt at once -> logits [T, vocab]; for prompts whose token-by-token run
    would take minutes."""
    w = {k: np.asarray(v, dtype=np.float64) for k, v in w.items()}
    eps, n = cfg["norm"]["eps"], len(tokens)
    x0 = w["embed"][np.asarray(tokens)]
    x = x0
    for L, t, first in schedule(cfg):
        if first:
            x = np.concatenate([x, x0], axis=1) @ w["loop.in"].T + w["loop.step"][t]
        p, layer = f"l{L}.", cfg["layers"][L]
        mix, m = layer["mixer"], p + "mix."
        nh, dim, rot, vdim, half = mix["heads"], mix["dim"], mix["rot_dim"], mix["vdim"], mix["rot"]["dims"] // 2
        angle = np.arange(n)[:, None] * float(mix["rot"]["base"]) ** (-2.0 * np.arange(half) / mix["rot"]["dims"])
        cos, sin = np.cos(angle), np.sin(angle)

        def turn(v):   # [T, ..., rot]
            c, s = (a.reshape((n,) + (1,) * (v.ndim - 2) + (half,)) for a in (cos, sin))
            a, b = v[..., :half], v[..., half:2 * half]
            return np.concatenate([a * c - b * s, b * c + a * s, v[..., 2 * half:]], axis=-1)

        h = norm(x, p + "norm1", w)
        q = (h @ w[m + "q"].T).reshape(n, nh, dim + rot)
        kv = h @ w[m + "dkv"].T
        c = rms_norm(kv[:, :mix["kv_rank"]], w[m + "dkv.norm"], eps)
        kr = turn(kv[:, mix["kv_rank"]:])
        qr = turn(q[..., dim:])
        outs = []
        for j in range(nh):
            s = (q[:, j, :dim] @ (c @ w[m + "uk"][j * dim:(j + 1) * dim].T).T + qr[:, j] @ kr.T) * mix["scale"]
            s = np.where(np.tril(np.ones((n, n), dtype=bool)), s, -np.inf)
            sink = float(w[m + "sink"][j])
            top = np.maximum(s.max(axis=1), sink)
            e = np.exp(s - top[:, None])
            outs.append((e / (e.sum(axis=1) + np.exp(sink - top))[:, None]) @ (c @ w[m + "uv"][j * vdim:(j + 1) * vdim].T))
        x = x + np.concatenate(outs, axis=1) @ w[m + "o"].T
        if layer.get("mlp"):
            x = x + gelu_tanh(norm(x, p + "norm2", w) @ w[p + "mlp.up"].T) @ w[p + "mlp.down"].T
    return norm(x, "final.norm", w) @ w["embed"].T * cfg["logit_scale"]
