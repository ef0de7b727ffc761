"""Host side of the Muvonex design, no GPU: configuration and its errors; the oracle's own consistency and the sensitivity
of the test weights (mistakes planted in the oracle must show)."""
from __future__ import annotations

import json

import numpy as np
import pytest

import muvonex_models as mm
from oracle import plain_muvonex as plain
from oxibonsai_amd import _lib
from oxibonsai_amd.backend import GpuError
from oxibonsai_amd.model import checkpoint_info


def info_of(tmp_path, text):
    (tmp_path / "config.json").write_text(text)
    return checkpoint_info(str(tmp_path))


def changed(**kw):
    cfg = json.loads(json.dumps(mm.MIXED))
    for path, value in kw.items():
        at, keys = cfg, path.split("__")
        for k in keys[:-1]:
            at = at[int(k)] if isinstance(at, list) else at[k]
        if value is KeyError:
            del at[keys[-1]]
        else:
            at[keys[-1]] = value
    return json.dumps(cfg)


def test_checkpoint_info(tmp_path):
    d = info_of(tmp_path, json.dumps(mm.MIXED))
    assert d["architecture"] == "Muvonex" and (d["n_layers"], d["n_runs"], d["h"], d["vocab"]) == (4, 4, 150, 131)
    for text in (changed(layers__0__mlp=None), changed(layers__0__mlp=KeyError), changed(layers__1__mixer__left__rot__scaling=None)):
        assert info_of(tmp_path, text)["n_layers"] == 4


@pytest.mark.parametrize("text,says", [
    (changed(residual_mult=KeyError), "residual_mult"), (changed(embedding=KeyError), "embedding"), (changed(embedding__scale="x"), "embedding.scale"),
    (changed(layers__0__type="latent_attention"), 'layers[0].type "latent_attention"'), (changed(layers__0__mixer__conv=0), "layers[0].mixer.conv"),
    (changed(layers__0__mixer__kv_heads=4), "kv_heads"), (changed(layers__0__mixer__vdim=KeyError), "layers[0].mixer.vdim"),
    (changed(layers__1__mixer__left__rot__dims=42), "left.rot.dims"), (changed(layers__1__mixer__left__rot__scaling__factor=0), "factor"),
    (changed(layers__1__mixer__left__rot__scaling__high=KeyError), "scaling.high"), (changed(layers__1__mixer__right__groups=3), "groups"),
    (changed(layers__1__mixer__right__norm_groups=7), "norm_groups"), (changed(layers__1__mixer__right=KeyError), "right"),
    (changed(layers__1__mixer__left_scale=KeyError), "left_scale"), (changed(layers__0__mlp__kind="routed"), 'layers[0].mlp.kind "routed"')])
def test_configuration_errors_name_the_key(tmp_path, text, says):
    with pytest.raises(GpuError) as e:
        info_of(tmp_path, text)
    assert says in str(e.value), str(e.value)


def test_oracle_portions():
    cfg = mm.MIXED
    w = mm.values(mm.weights(cfg, 2))
    ids = mm.tokens(cfg, 3, 14)
    t = plain.run(cfg, w, ids)
    s = plain.Sequence(cfg, w)
    assert np.allclose(np.concatenate([s.step(ids[:9]), s.step(ids[9:11]), s.step(ids[11:])]), t.logits, atol=1e-12)
    assert t.layers.shape == (4, 14, cfg["width"])


def test_oracle_mechanisms():
    """Hand-checked values and invariants of the oracle's functions."""
    assert np.allclose(plain.rms(np.array([3.0, 4.0]), 0.0), np.array([3.0, 4.0]) / np.sqrt(12.5))
    assert np.allclose(plain.zero_centred_norm(np.array([1.0, -1.0]), np.array([0.0, 0.5]), 0.0), [1.0, -1.5])
    assert np.allclose(plain.gelu_tanh(np.array([0.0, 1.0, -1.0])), [0.0, 0.8411919906, -0.1588080094], atol=1e-9)
    assert np.allclose([plain.softplus(0.0), plain.softplus(100.0), plain.silu(0.0), plain.sigmoid(0.0)], [np.log(2.0), 100.0, 0.0, 0.5])
    assert np.allclose(plain.unit(np.array([3.0, 4.0])), [0.6, 0.8], atol=1e-7) and np.allclose(plain.unit(np.zeros(3)), 0)
    p = plain.softmax_with_sink(np.array([0.0, 0.0]), 0.0)
    assert np.allclose(p, 1 / 3) and np.allclose(plain.softmax_with_sink(np.array([800.0, 0.0]), -5.0), [1, 0])
    rot = {"base": 100.0, "dims": 4}
    v = np.arange(1.0, 7.0)
    r = plain.rotate_half(v, 3, rot)
    assert np.allclose(r[[0, 2]], [np.cos(3) - 3 * np.sin(3), 3 * np.cos(3) + np.sin(3)]) and np.allclose(r[4:], v[4:])
    # scaled frequencies: short turns stay, long turns slow down by the factor, between them a blend
    rot = {"base": 1e4, "dims": 16, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 200}}
    f = [plain.frequency(i, rot) for i in range(8)]
    g = [1e4 ** (-i / 8) for i in range(8)]
    turn = [2 * np.pi / x for x in g]
    assert [x == y for x, y in zip(f, g)] == [t < 50 for t in turn]
    assert all(np.isclose(x, y / 8) == (t > 200) for x, y, t in zip(f, g, turn)) and any(50 < t < 200 for t in turn)
    # delta rule: with decay and beta one a written key reads back its value, a second write replaces it
    k = plain.unit(np.array([1.0, 2.0, -1.0]))
    s, _ = plain.delta_update(np.zeros((3, 2)), 1.0, 1.0, k, k, np.array([5.0, 7.0]))
    s, o = plain.delta_update(s, 1.0, 1.0, k, k, np.array([1.0, -1.0]))
    assert np.allclose(o, [1.0, -1.0], atol=1e-5)
    s, o = plain.ssd_update(np.ones((2, 1)), 0.5, 2.0, np.array([3.0]), np.array([1.0, 0.0]), np.array([1.0, 1.0]), 10.0)
    assert np.allclose(s[:, 0], [6.5, 0.5]) and np.allclose(o, [37.0])
    c = plain.Window(3, 1)
    w = np.array([[1.0, 10.0, 100.0]])
    assert [float(plain.short_conv(c.push(np.array([x])), w)[0]) for x in (1.0, 2.0, 3.0)] == [100.0, 210.0, 321.0]


def sequence_with(**kw):
    """Sequence whose memory is tampered with behind every token: kw maps 'conv' / 's' / 'kv' to a function."""
    class Tampered(plain.Sequence):
        def token(self, tok):
            out = super().token(tok)
            for memory in self.memory:
                for k, f in kw.items():
                    f(self, memory)
            return out
    return Tampered


def lose_state(seq, memory):
    if seq.position == 20 and "s" in memory:
        memory["s"][:] = 0


def lose_window(seq, memory):
    if seq.position == 20:
        for v in memory.values():
            if isinstance(v, plain.Window):
                v.past[:] = 0


def lose_oldest_tap(seq, memory):
    for v in memory.values():
        if isinstance(v, plain.Window) and len(v.past):
            v.past[0] = 0


@pytest.mark.parametrize("mistake", ["no sink", "sink twice", "scaled sink", "no rotation", "rotation one off", "interleaved pairs", "unscaled frequencies",
                                     "unnormed heads", "wrong group", "write after read", "no decay", "decay after", "no beta", "gate after norm", "no skip",
                                     "clamped step", "norm weight one off", "no unit", "state lost", "window lost", "oldest tap", "silu before"])
def test_mistakes_show(monkeypatch, mistake):
    """The weights the GPU tests use expose each of these mistakes by more than their bf16 tolerance allows."""
    cfg = mm.MIXED
    w = mm.values(mm.weights(cfg, 21))
    ids = mm.tokens(cfg, 22, 40)
    want = plain.run(cfg, w, ids).logits
    softmax, rotate, att, rms = plain.softmax_with_sink, plain.rotate_half, plain.grouped_attention, plain.rms
    put = monkeypatch.setattr
    if mistake == "no sink":
        put(plain, "softmax_with_sink", lambda s, k: softmax(s, -1e9))
    elif mistake == "sink twice":
        put(plain, "softmax_with_sink", lambda s, k: softmax(s, k + np.log(2)))
    elif mistake == "scaled sink":
        put(plain, "softmax_with_sink", lambda s, k: softmax(s, 0.2 * k))
    elif mistake == "no rotation":
        put(plain, "rotate_half", lambda v, pos, rot: v)
    elif mistake == "rotation one off":   # keys alone: a common shift would cancel
        put(plain, "rotate_half", lambda v, pos, rot: rotate(v, pos + (v.shape[0] in (1, 2)), rot))
    elif mistake == "interleaved pairs":
        def pairs(v, pos, rot):
            d = rot["dims"]
            order = np.r_[np.arange(0, d, 2), np.arange(1, d, 2), np.arange(d, v.shape[-1])]
            out = np.empty_like(v)
            out[..., order] = rotate(v[..., order], pos, rot)
            return out
        put(plain, "rotate_half", pairs)
    elif mistake == "unscaled frequencies":
        put(plain, "frequency", lambda i, rot: float(rot["base"]) ** (-2.0 * i / rot["dims"]))
    elif mistake == "unnormed heads":
        put(plain, "rms", lambda x, eps: x if x.ndim == 2 and x.shape[-1] in (40, 16) else rms(x, eps))
    elif mistake == "wrong group":
        def turned(h, position, history, mix, p, wts, eps):
            k = wts[p + "k"].reshape(mix["kv_heads"], -1)
            return att(h, position, history, mix, p, dict(wts, **{p + "k": np.roll(k, 1, 0).reshape(wts[p + "k"].shape)}), eps)
        put(plain, "grouped_attention", turned)
    elif mistake == "write after read":
        def late(s, a, beta, q, k, v):
            s = a * s
            o = s.T @ q
            return s + np.outer(k, beta * (v - s.T @ k)), o
        put(plain, "delta_update", late)
    elif mistake == "no decay":
        update = plain.delta_update
        put(plain, "delta_update", lambda s, a, *r: update(s, 1.0, *r))
    elif mistake == "decay after":
        def after(s, a, beta, q, k, v):
            s = s + np.outer(k, beta * (v - s.T @ k))
            return a * s, a * s.T @ q
        put(plain, "delta_update", after)
    elif mistake == "no beta":
        update = plain.delta_update
        put(plain, "delta_update", lambda s, a, beta, *r: update(s, a, 1.0, *r))
    elif mistake == "gate after norm":
        space = plain.state_space

        def ungated(h, memory, mix, p, wts, eps):
            z = wts[p + "in"][:mix["heads"] * mix["vdim"]] @ h
            calls = []

            def gate(x):
                calls.append(x)
                return np.ones_like(x) if len(calls) == 2 else x / (1.0 + np.exp(-x))
            put(plain, "silu", gate)
            out = space(h, memory, mix, p, dict(wts, **{p + "norm": wts[p + "norm"] * (z / (1.0 + np.exp(-z)))}), eps)
            put(plain, "silu", lambda x: x / (1.0 + np.exp(-x)))
            return out
        put(plain, "state_space", ungated)
    elif mistake == "no skip":
        update = plain.ssd_update
        put(plain, "ssd_update", lambda s, a, dt, x, b, c, d: update(s, a, dt, x, b, c, 0.0))
    elif mistake == "clamped step":
        put(plain, "softplus", lambda z: np.minimum(np.logaddexp(0.0, z), 0.5))
    elif mistake == "norm weight one off":
        put(plain, "zero_centred_norm", lambda x, wt, eps: rms(x, eps) * wt)
    elif mistake == "no unit":
        put(plain, "unit", lambda x: x)
    elif mistake == "silu before":
        conv = plain.short_conv
        put(plain, "short_conv", lambda x, wt, bias=0.0: conv(plain.silu(x), wt, bias))
    else:
        f = {"state lost": lose_state, "window lost": lose_window, "oldest tap": lose_oldest_tap}[mistake]
        put(plain, "Sequence", sequence_with(m=f))
    with np.errstate(all="ignore"):
        got = plain.run(cfg, w, ids).logits
    assert not np.all(np.isfinite(got)) or mm.error(got, want) > 0.12, mm.error(got, want)


def test_checkpoint_errors_before_a_gpu_is_needed(tmp_path):
    import ctypes as C
    (tmp_path / "config.json").write_text(json.dumps(mm.PLAIN))
    mid, eid = C.c_uint64(0), C.c_uint64(0)
    rc = _lib.lib().oxb_hip_load_checkpoint(str(tmp_path).encode(), 0, 64, 1, C.byref(mid), C.byref(eid), None)
    assert rc == 5 and "cannot open" in _lib.last_error()
