"""Small Fulirax configurations and random weights for the tests; weights are bfloat16 bit patterns, as checkpoints hold
them, and the oracle gets exactly the values they stand for."""
from __future__ import annotations

import copy
import json
import struct

import numpy as np


def bf16_bits(a) -> np.ndarray:
    """float -> bfloat16 bit pattern, round to nearest even."""
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32).astype(np.uint64)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16).reshape(np.shape(a))


def bf16_value(bits) -> np.ndarray:
    return (np.atleast_1d(np.asarray(bits, dtype=np.uint32)) << 16).view(np.float32).reshape(np.shape(bits))


def layer(heads, dim, rot_dim, vdim, kv_rank, ff=0, base=10000.0, scale=None, rot_dims=None):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
                      "rot": {"base": base, "dims": rot_dims or rot_dim}, "scale": scale or (dim + rot_dim) ** -0.5},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(width, vocab, layers, loop=None, eps=1e-5, logit_scale=0.7):
    return {"architecture": "Fulirax", "width": width, "vocab": vocab, "layers": copy.deepcopy(layers),
            "loop": dict(zip(("start", "stop", "times"), loop)) if loop else None, "norm": {"eps": eps}, "logit_scale": logit_scale}


# sizes that differ from layer to layer, none a multiple of the kernels' tiles; a repeated range that starts behind the
# first layer; one layer without a feed-forward
MIXED = config(150, 131, [layer(5, 24, 8, 40, 72, ff=200), layer(17, 16, 32, 20, 48, base=500.0), layer(3, 40, 12, 28, 100, ff=90)],
               loop=(1, 3, 2))
# one head, no loop
PLAIN = config(96, 70, [layer(1, 64, 16, 64, 64, ff=128), layer(2, 20, 6, 10, 33, ff=77)])
# a loop over everything, once
ONCE = config(64, 90, [layer(2, 32, 16, 48, 96, ff=64), layer(2, 32, 16, 48, 96, ff=64)], loop=(0, 2, 1))
# latents as long as a large model's
WIDE = config(128, 64, [layer(18, 128, 64, 128, 512, ff=160), layer(2, 48, 24, 16, 640)], loop=(0, 1, 2))


def weights(cfg, seed, sharp=1.0, sink=1.0):
    """name -> bfloat16 bits.  `sharp` scales the queries, so that single keys stand out of a long context."""
    rng = np.random.default_rng(seed)
    w, out = cfg["width"], {}

    def put(name, *shape, std=1.0, mean=0.0):
        out[name] = bf16_bits(rng.normal(mean, std, shape))

    def norm(name):
        put(name, w, std=0.2, mean=1.0)
        put(name + ".b", w, std=0.2)
        put(name + ".alpha", std=0.15, mean=0.6)

    put("embed", cfg["vocab"], w)
    if cfg.get("loop"):
        put("loop.in", w, 2 * w, std=0.7 * (2 * w) ** -0.5)
        put("loop.step", cfg["loop"]["times"], w, std=0.3)
    for i, layer_ in enumerate(cfg["layers"]):
        m, p = layer_["mixer"], f"l{i}."
        norm(p + "norm1")
        put(p + "mix.q", m["heads"] * (m["dim"] + m["rot_dim"]), w, std=1.5 * sharp * w ** -0.5)
        put(p + "mix.dkv", m["kv_rank"] + m["rot_dim"], w, std=1.5 * w ** -0.5)
        dkv = bf16_value(out[p + "mix.dkv"])
        dkv[m["kv_rank"]:] *= 3.0   # (rotation has to matter beside the unrotated scores)
        out[p + "mix.dkv"] = bf16_bits(dkv)
        put(p + "mix.dkv.norm", m["kv_rank"], std=0.2, mean=1.0)
        put(p + "mix.uk", m["heads"] * m["dim"], m["kv_rank"], std=m["kv_rank"] ** -0.5)
        put(p + "mix.uv", m["heads"] * m["vdim"], m["kv_rank"], std=m["kv_rank"] ** -0.5)
        put(p + "mix.sink", m["heads"], std=sink, mean=sink)
        put(p + "mix.o", w, m["heads"] * m["vdim"], std=(m["heads"] * m["vdim"]) ** -0.5)
        if layer_["mlp"]:
            norm(p + "norm2")
            put(p + "mlp.up", layer_["mlp"]["ff"], w, std=w ** -0.5)
            put(p + "mlp.down", w, layer_["mlp"]["ff"], std=layer_["mlp"]["ff"] ** -0.5)
    norm("final.norm")
    return out


def values(bits: dict) -> dict:
    return {k: bf16_value(v) for k, v in bits.items()}


def write_checkpoint(folder, cfg, bits) -> str:
    header, blob = {}, b""
    for name, a in bits.items():
        raw = np.asarray(a, dtype="<u2").tobytes()
        header[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [len(blob), len(blob) + len(raw)]}
        blob += raw
    head = json.dumps(header).encode()
    (folder / "config.json").write_text(json.dumps(cfg))
    (folder / "model.safetensors").write_bytes(struct.pack("<Q", len(head)) + head + blob)
    return str(folder)


def tokens(cfg, seed, n):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


def rms(a) -> float:
    return float(np.sqrt(np.mean(np.square(np.asarray(a, dtype=np.float64)))))


def error(got, want) -> float:
    """Largest RMS difference of a row of logits, in units of the logits' own spread."""
    d = np.asarray(got, dtype=np.float64) - want
    return float(np.max(np.sqrt(np.mean(d * d, axis=-1)))) / float(np.std(want))
