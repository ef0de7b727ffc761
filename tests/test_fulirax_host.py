"""Host side of configured designs, no GPU: registry, configuration and checkpoint errors; the oracle's own consistency and
the sensitivity of the test weights (mistakes planted in the oracle must show)."""
from __future__ import annotations

import json
import struct

import numpy as np
import pytest

import fulirax_models as fm
from oracle import plain_fulirax as plain
from oxibonsai_amd import _lib
from oxibonsai_amd.backend import GpuError
from oxibonsai_amd.model import checkpoint_info


def info_of(tmp_path, text):
    (tmp_path / "config.json").write_text(text)
    return checkpoint_info(str(tmp_path))


def changed(**kw):
    cfg = json.loads(json.dumps(fm.MIXED))
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
    d = info_of(tmp_path, json.dumps(fm.MIXED))
    assert d["architecture"] == "Fulirax" and (d["n_layers"], d["n_runs"], d["h"], d["vocab"]) == (3, 5, 150, 131)
    assert info_of(tmp_path, changed(loop=None))["n_runs"] == 3
    assert info_of(tmp_path, changed(loop=KeyError))["n_runs"] == 3
    assert info_of(tmp_path, changed(loop={"start": 0, "stop": 3, "times": 4}))["n_runs"] == 12
    assert info_of(tmp_path, changed(layers__0__mlp=KeyError))["n_runs"] == 5


@pytest.mark.parametrize("text,says", [
    (changed(architecture="Nothing"), "unknown (known: Fulirax"), (changed(architecture=KeyError), "architecture is missing"),
    (changed(width=0), "width"), (changed(vocab=1.5), "vocab"), (changed(layers=[]), "layers"),
    (changed(layers__1__type="mystery"), 'layers[1].type "mystery"'), (changed(layers__2__mixer__kv_rank=KeyError), "layers[2].mixer.kv_rank"),
    (changed(layers__0__mlp__kind="routed"), 'layers[0].mlp.kind "routed"'), (changed(layers__0__mixer__rot__dims=7), "rot.dims"),
    (changed(layers__0__mixer__rot__dims=10), "rot.dims"), (changed(loop__stop=4), "loop.stop"), (changed(loop__start=3), "loop"),
    (changed(loop__times=0), "loop.times"), (changed(norm=KeyError), "norm"), (changed(logit_scale="1"), "logit_scale"),
    ("{", "byte"), ("[1, 2]", "architecture"), ('{"a": 1} x', "text after"), ('{"a": "\\q"}', "escape"), ("[" * 100, "deep"), ("", "end")])
def test_configuration_errors_name_the_key(tmp_path, text, says):
    with pytest.raises(GpuError) as e:
        info_of(tmp_path, text)
    assert says in str(e.value), str(e.value)


def test_json_values(tmp_path):
    text = json.dumps(fm.PLAIN, indent=1).replace('"Fulirax"', '"\\u0046ulirax"').replace("70", "7.0e1") + "\n"
    d = info_of(tmp_path, text)
    assert d["architecture"] == "Fulirax" and d["vocab"] == 70


def load(path, dtype=0):
    import ctypes as C
    mid, eid = C.c_uint64(0), C.c_uint64(0)
    rc = _lib.lib().oxb_hip_load_checkpoint(str(path).encode(), dtype, 64, 1, C.byref(mid), C.byref(eid), None)
    return rc, _lib.last_error()


def test_checkpoint_file_errors(tmp_path):
    """Each is found while the file is read, before a GPU is needed."""
    fm.write_checkpoint(tmp_path, fm.PLAIN, fm.weights(fm.PLAIN, 1))
    f = tmp_path / "model.safetensors"
    good = f.read_bytes()
    n = struct.unpack("<Q", good[:8])[0]

    def with_header(edit):
        h = json.loads(good[8:8 + n])
        edit(h)
        t = json.dumps(h).encode()
        return struct.pack("<Q", len(t)) + t + good[8 + n:]

    def entry(**kw):
        return lambda h: h["embed"].update(kw)

    for data, says in ((good[:4], "end of file"), (struct.pack("<Q", 1 << 60) + good[8:], "does not fit"), (good[:8] + b"x" * 40, "header"),
                       (good[:8 + n], "outside the file"), (with_header(entry(shape=[1, 2])), "embed"), (with_header(entry(shape=[-1])), "embed"),
                       (with_header(entry(data_offsets=[8, 4])), "embed"), (with_header(entry(shape="x")), "embed")):
        f.write_bytes(data)
        rc, why = load(tmp_path)
        assert rc == 5 and says in why, (says, why)
    f.unlink()
    rc, why = load(tmp_path)
    assert rc == 5 and "cannot open" in why
    rc, why = load(tmp_path / "nowhere.gguf")
    assert rc == 5


def test_oracle_portions_and_schedule():
    cfg = fm.MIXED
    w = fm.values(fm.weights(cfg, 2))
    ids = fm.tokens(cfg, 3, 14)
    t = plain.run(cfg, w, ids)
    s = plain.Sequence(cfg, w)
    assert np.allclose(np.concatenate([s.step(ids[:9]), s.step(ids[9:11]), s.step(ids[11:])]), t.logits, atol=1e-12)
    assert plain.schedule(cfg) == [(0, None, False), (1, 0, True), (2, 0, False), (1, 1, True), (2, 1, False)]
    assert t.layers.shape == (5, 14, cfg["width"])


def test_oracle_matrix_form():
    for cfg in (fm.MIXED, fm.PLAIN):
        w = fm.values(fm.weights(cfg, 4))
        ids = fm.tokens(cfg, 5, 25)
        assert np.allclose(plain.run_prompt(cfg, w, ids), plain.run(cfg, w, ids).logits, atol=1e-10)


def test_oracle_mechanisms():
    """Hand-checked values and invariants of the oracle's functions."""
    assert np.allclose(plain.dynamic_tanh(np.array([0.0, 1e9, -1e9]), 0.5, np.array([2.0, 2.0, 2.0]), np.array([1.0, 1.0, 1.0])), [1.0, 3.0, -1.0])
    assert np.allclose(plain.gelu_tanh(np.array([0.0, 1.0, -1.0, 30.0])), [0.0, 0.8411919906, -0.1588080094, 30.0], atol=1e-9)
    v = np.arange(1.0, 7.0)
    r = plain.rotate_half(v, 3, 100.0, 4)   # pairs (0, 2) and (1, 3); elements 4, 5 stay
    assert np.allclose(r[[0, 2]], [np.cos(3) - 3 * np.sin(3), 3 * np.cos(3) + np.sin(3)]) and np.allclose(r[4:], v[4:])
    assert np.allclose(r[1], 2 * np.cos(0.3) - 4 * np.sin(0.3))
    p = plain.softmax_with_sink(np.array([0.0, 0.0]), 0.0)
    assert np.allclose(p, 1 / 3) and np.allclose(plain.softmax_with_sink(np.array([800.0, 0.0]), -5.0), [1, 0])
    assert np.allclose(plain.rms_norm(np.array([3.0, 4.0]), np.array([1.0, 2.0]), 0.0), np.array([3.0, 8.0]) / np.sqrt(12.5))


@pytest.mark.parametrize("mistake", ["no sink", "sink twice", "no rotation", "rotation one off", "no loop entry", "stale pass", "interleaved pairs",
                                     "scaled sink", "unnormed latent", "rotated unrotated"])
def test_mistakes_show(monkeypatch, mistake):
    """The weights the GPU tests use expose each of these mistakes by more than their bf16 tolerance allows."""
    cfg = fm.MIXED
    w = fm.values(fm.weights(cfg, 21))
    ids = fm.tokens(cfg, 22, 40)
    want = plain.run(cfg, w, ids).logits
    softmax, rotate, rms, entry, latent = plain.softmax_with_sink, plain.rotate_half, plain.rms_norm, plain.loop_entry, plain.latent_entry
    sequence = plain.Sequence
    if mistake == "no sink":
        monkeypatch.setattr(plain, "softmax_with_sink", lambda s, k: softmax(s, -1e9))
    elif mistake == "sink twice":
        monkeypatch.setattr(plain, "softmax_with_sink", lambda s, k: softmax(s, k + np.log(2)))
    elif mistake == "scaled sink":
        monkeypatch.setattr(plain, "softmax_with_sink", lambda s, k: softmax(s, 0.2 * k))
    elif mistake == "no rotation":
        monkeypatch.setattr(plain, "rotate_half", lambda v, pos, base, dims: v)
    elif mistake == "rotation one off":   # keys alone: a common shift would cancel
        monkeypatch.setattr(plain, "latent_entry", lambda h, pos, *a: latent(h, pos + 1, *a))
    elif mistake == "interleaved pairs":
        def pairs(v, pos, base, dims):
            i = np.argsort(np.r_[np.arange(0, dims, 2), np.arange(1, dims, 2)])
            half = np.r_[np.arange(0, dims, 2), np.arange(1, dims, 2), np.arange(dims, len(v))]
            out = rotate(v[half], pos, base, dims)
            return np.r_[out[:dims][i], out[dims:]]
        monkeypatch.setattr(plain, "rotate_half", pairs)
    elif mistake == "unnormed latent":
        monkeypatch.setattr(plain, "rms_norm", lambda x, wt, eps: x * wt)
    elif mistake == "rotated unrotated":
        monkeypatch.setattr(plain, "latent_entry", lambda h, pos, *a: (rotate(latent(h, pos, *a)[0], pos, 100.0, 16), latent(h, pos, *a)[1]))
    elif mistake == "no loop entry":
        monkeypatch.setattr(plain, "loop_entry", lambda x, x0, t, wts: x)
    elif mistake == "stale pass":   # later passes read the first pass's history
        class Shared(sequence):
            def __init__(self, c, wts):
                super().__init__(c, wts)
                for r, (L, t, _) in enumerate(self.runs):
                    if t:
                        self.history[r] = self.history[[q for q, x in enumerate(self.runs) if x[0] == L][0]]
        monkeypatch.setattr(plain, "Sequence", Shared)
    assert fm.error(plain.run(cfg, w, ids).logits, want) > 0.12, fm.error(plain.run(cfg, w, ids).logits, want)
