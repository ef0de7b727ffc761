"""Small Muvonex configurations and random weights for the tests; weights are bfloat16 bit patterns, as checkpoints hold
them, and the oracle gets exactly the values they stand for."""
from __future__ import annotations

import copy

import numpy as np

from fulirax_models import bf16_bits, bf16_value, error, tokens, values, write_checkpoint  # noqa: F401


def mlp(ff):
    return {"kind": "dense", "ff": ff} if ff else None


def delta(heads, kv_heads, dim, vdim, conv=4, ff=0):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, "mlp": mlp(ff)}


def attention(heads, kv_heads, dim, vdim, rot_dims=None, base=10000.0, scaling=None, scale=None):
    rot = {"base": base, "dims": rot_dims or dim - dim % 2}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "rot": rot, "scale": scale or dim ** -0.5}


def space(heads, vdim, state, groups=1, norm_groups=1, conv=4):
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups, "conv": conv}


def parallel(left, right, left_scale=0.8, right_scale=0.55, ff=0):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}, "mlp": mlp(ff)}


def config(width, vocab, layers, eps=1e-5, embed_scale=1.5, residual_mult=0.7):
    return {"architecture": "Muvonex", "width": width, "vocab": vocab, "layers": copy.deepcopy(layers), "norm": {"eps": eps},
            "embedding": {"scale": embed_scale}, "residual_mult": residual_mult}


# sizes that differ from layer to layer, hardly one a multiple of the kernels' tiles; layers with and without a feed-forward;
# convolutions of one to six taps; norm parts that cut across heads
MIXED = config(150, 131, [
    delta(6, 2, 24, 40, conv=3, ff=200),
    parallel(attention(6, 2, 40, 24, rot_dims=24, base=500.0, scaling=(8.0, 1.0, 4.0, 60)), space(4, 20, 12, groups=2, norm_groups=2, conv=6)),
    delta(3, 3, 50, 18, conv=1, ff=90),
    parallel(attention(5, 1, 16, 36), space(6, 10, 40, groups=3, norm_groups=4, conv=4), left_scale=1.1, right_scale=0.3, ff=77)])
# one head of everything
PLAIN = config(96, 70, [parallel(attention(1, 1, 32, 32), space(1, 32, 16), left_scale=1.0, right_scale=1.0, ff=128), delta(1, 1, 32, 32, ff=64)],
               embed_scale=1.0, residual_mult=1.0)
# heads as large as a large model's
WIDE = config(128, 64, [delta(4, 2, 128, 128, ff=160),
                        parallel(attention(20, 1, 128, 96, scaling=(4.0, 1.0, 4.0, 512)), space(4, 64, 128, groups=2), ff=96),
                        delta(2, 1, 200, 250)])


def weights(cfg, seed, memory=1.0, sink=1.0):
    """name -> bfloat16 bits.  `memory` divides the recurrences' decay rates: the larger, the longer they remember."""
    rng = np.random.default_rng(seed)
    w, out = cfg["width"], {}

    def put(name, *shape, std=1.0, mean=0.0):
        out[name] = bf16_bits(rng.normal(mean, std, shape))

    def linear(name, n, k, gain=1.0):
        put(name, n, k, std=gain * k ** -0.5)

    put("embed", cfg["vocab"], w, std=0.6)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        put(f"l{i}.norm1", w, std=0.2)
        if layer["type"] == "delta":
            qk, inner = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            for t, n in (("q", qk), ("k", qk), ("v", inner)):
                linear(p + t, n, w, 1.5)
                put(p + t + ".conv", n, m["conv"], std=0.6)
            linear(p + "b", m["heads"], w, 1.5)
            linear(p + "a", m["heads"], w)
            put(p + "A_log", m["heads"], std=0.5, mean=-2.0 - np.log(memory))
            put(p + "dt_bias", m["heads"], std=0.5)
            put(p + "norm", m["vdim"], std=0.2, mean=1.0)
            linear(p + "g", inner, w, 1.5)
            linear(p + "o", w, inner, 2.0)
        else:
            a, s = m["left"], m["right"]
            linear(p + "left.q", a["heads"] * a["dim"], w)
            linear(p + "left.k", a["kv_heads"] * a["dim"], w)
            linear(p + "left.v", a["kv_heads"] * a["vdim"], w, 1.5)
            put(p + "left.sink", a["heads"], std=sink, mean=1.5 * sink)
            linear(p + "left.o", w, a["heads"] * a["vdim"], 4.0)
            inner, gn = s["heads"] * s["vdim"], s["groups"] * s["state"]
            linear(p + "right.in", 2 * inner + 2 * gn + s["heads"], w, 1.5)
            put(p + "right.conv", inner + 2 * gn, s["conv"], std=0.6)
            put(p + "right.conv.b", inner + 2 * gn, std=0.3)
            put(p + "right.dt_bias", s["heads"], std=0.5, mean=-0.5)
            put(p + "right.A_log", s["heads"], std=0.5, mean=-1.5 - np.log(memory))
            put(p + "right.D", s["heads"], std=0.5, mean=0.5)
            put(p + "right.norm", inner, std=0.2, mean=1.0)
            linear(p + "right.o", w, inner, 1.5)
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            linear(f"l{i}.mlp.gate", ff, w, 1.5)
            linear(f"l{i}.mlp.up", ff, w, 1.5)
            linear(f"l{i}.mlp.down", w, ff, 1.5)
    put("final.norm", w, std=0.2)
    return out


def without(bits, *ends):
    """The weights with every tensor whose name ends so set to zero: what it feeds is switched off."""
    return {k: (np.zeros_like(v) if k.endswith(ends) else v) for k, v in bits.items()}


def scaled(bits, name, gain):
    return dict(bits, **{name: bf16_bits(bf16_value(bits[name]) * gain)})
