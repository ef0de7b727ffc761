"""Muvonex on the GPU against its plain oracle (oracle/plain_muvonex.py): mechanisms alone, prompts, portions, decoding,
batches, pages and slots, greedy generation; fp32 within rounding of 32 bits, bf16 within rounding of its products."""
from __future__ import annotations

import json
import os
import subprocess
import sys

import numpy as np
import pytest

import muvonex_models as mm
from oracle import plain_muvonex as plain

pytestmark = pytest.mark.gpu

TOL = {"float32": 3e-5, "bfloat16": 6e-2}
DTYPES = ["float32", "bfloat16"]


@pytest.fixture
def make(backend):
    """(cfg, bits, dtype, **kw) -> (model, embedding), closed at the end of the test."""
    from oxibonsai_amd.model import HipModel
    live = []

    def build(cfg, bits, dtype="float32", max_seq=256, batch=1):
        m, e = HipModel.from_tensors(backend, cfg, bits, dtype, max_seq=max_seq, batch=batch)
        live.extend([e, m])
        return m, e

    yield build
    for x in live:
        x.close()


def reference(cfg, bits, ids):
    return plain.run(cfg, mm.values(bits), ids).logits


def whole(m, e, ids, seq=0):
    return m.forward_tokens(e, ids, 0, seq, want=range(len(ids)))


def in_portions(m, e, ids, sizes, seq=0, at=0):
    """The tokens from place `at` on, cut into portions of the given sizes, cyclically."""
    out, k = [], 0
    while at < len(ids):
        n = min(sizes[k % len(sizes)], len(ids) - at)
        out.append(m.forward_tokens(e, ids[at:at + n], at, seq, want=range(n)))
        at, k = at + n, k + 1
    return np.concatenate(out)


# --- mechanisms alone: everything else is switched off through the weights -------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,scale", [(90, 0.01), (90, 1.0), (6000, 30.0)])
def test_norm_and_embedding_scale_alone(make, dtype, width, scale):
    """Small streams too, where eps decides; a row longer than a workgroup keeps in registers."""
    cfg = mm.config(width, 77, [mm.delta(1, 1, 8, 8)], eps=1e-3, embed_scale=scale)
    bits = mm.without(mm.weights(cfg, 1), "mix.o")
    ids = mm.tokens(cfg, 2, 40)
    m, e = make(cfg, bits, dtype)
    w = {k: v.astype(np.float64) for k, v in mm.values(bits).items()}
    want = plain.zero_centred_norm(w["embed"][ids] * scale, w["final.norm"], 1e-3) @ w["embed"].T
    assert mm.error(whole(m, e, ids), want) < (2e-6 if dtype == "float32" else 1e-2)
    assert mm.error(in_portions(m, e, ids[:5], [1]), want[:5]) < (2e-6 if dtype == "float32" else 1e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [1, 133, 2000])
@pytest.mark.parametrize("gain", [0.02, 1.0, 8.0])
def test_gated_feed_forward_alone(make, dtype, ff, gain):
    cfg = mm.config(72, 50, [mm.delta(1, 1, 8, 8, ff=ff)], residual_mult=1.3)
    bits = mm.without(mm.weights(cfg, 3), "mix.o")
    bits = mm.scaled(mm.scaled(bits, "l0.mlp.gate", gain), "l0.mlp.down", 2.0 / gain)
    ids = mm.tokens(cfg, 4, 130)
    m, e = make(cfg, bits, dtype)
    w = {k: v.astype(np.float64) for k, v in mm.values(bits).items()}
    x = w["embed"][ids] * cfg["embedding"]["scale"]
    h = plain.zero_centred_norm(x, w["l0.norm1"], 1e-5)
    x = x + 1.3 * (plain.gelu_tanh(h @ w["l0.mlp.gate"].T) * (h @ w["l0.mlp.up"].T)) @ w["l0.mlp.down"].T
    want = plain.zero_centred_norm(x, w["final.norm"], 1e-5) @ w["embed"].T
    for n in (130, 20, 7):
        assert mm.error(whole(m, e, ids[:n]), want[:n]) < (5e-6 if dtype == "float32" else 3e-2), n


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(3, 3, 16, 24), (8, 2, 72, 40), (20, 1, 34, 130), (2, 2, 256, 8), (4, 2, 6, 256)])
def test_grouped_attention_alone(make, dtype, heads, kv_heads, dim, vdim):
    cfg = mm.config(64, 40, [mm.parallel(mm.attention(heads, kv_heads, dim, vdim, scale=0.4), mm.space(1, 8, 8))])
    bits = mm.without(mm.weights(cfg, 5), "right.o")
    ids = mm.tokens(cfg, 6, 75)
    m, e = make(cfg, bits, dtype)
    want = reference(cfg, bits, ids)
    assert mm.error(whole(m, e, ids), want) < TOL[dtype]
    assert mm.error(in_portions(m, e, ids, [33, 2, 9, 1]), want) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sink", [-40.0, 0.0, 4.0, 30.0])
@pytest.mark.parametrize("n", [1, 3, 40])
def test_sink(make, dtype, sink, n):
    """From a sink that takes nothing to one that takes everything; decided alone (n = 1), in a short portion, in a prompt."""
    cfg = mm.config(64, 40, [mm.parallel(mm.attention(3, 1, 16, 24), mm.space(1, 8, 8))])
    bits = mm.without(mm.weights(cfg, 7), "right.o")
    bits["l0.mix.left.sink"] = mm.bf16_bits([sink, sink + 1.0, sink - 2.0])
    ids = mm.tokens(cfg, 8, n)
    m, e = make(cfg, bits, dtype)
    want = reference(cfg, bits, ids)
    assert mm.error(whole(m, e, ids), want) < TOL[dtype]
    assert mm.error(in_portions(m, e, ids, [1]), want) < TOL[dtype]


@pytest.mark.parametrize("rot", [dict(rot_dims=24, base=30.0), dict(rot_dims=10, base=30.0), dict(base=500.0, scaling=(6.0, 1.0, 4.0, 60)),
                                 dict(rot_dims=16, base=1e5, scaling=(2.0, 0.5, 9.0, 300)), dict(base=100.0, scaling=(1.0, 1.0, 1.0, 50))])
def test_rotation_and_its_scaling(make, rot):
    """Positions matter through rotated dimensions that may be fewer than the head's; each scaling has fast, slow and blended
    pairs, or none between."""
    cfg = mm.config(80, 30, [mm.parallel(mm.attention(2, 1, 24, 16, scale=1.5, **rot), mm.space(1, 8, 8))])
    bits = mm.without(mm.weights(cfg, 9), "right.o")
    ids = [3] * 4 + mm.tokens(cfg, 10, 150)
    m, e = make(cfg, bits)
    want = reference(cfg, bits, ids)
    assert mm.error(whole(m, e, ids), want) < TOL["float32"]
    other = json.loads(json.dumps(cfg))
    r = other["layers"][0]["mixer"]["left"]["rot"]
    r["base"] *= 1.1
    assert mm.error(reference(other, bits, ids), want) > 1e-2
    if r.get("scaling", {}).get("factor", 1.0) != 1.0:
        other = json.loads(json.dumps(cfg))
        other["layers"][0]["mixer"]["left"]["rot"]["scaling"]["factor"] *= 2.0
        assert mm.error(reference(other, bits, ids), want) > 1e-2


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("space", [mm.space(1, 8, 8, conv=1), mm.space(6, 20, 40, groups=3, norm_groups=8, conv=2), mm.space(8, 64, 128, groups=2, norm_groups=1, conv=4),
                                   mm.space(4, 100, 16, groups=4, norm_groups=4, conv=9), mm.space(2, 256, 200, groups=1, norm_groups=1), mm.space(3, 7, 65, norm_groups=7)])
def test_state_space_alone(make, dtype, space):
    cfg = mm.config(64, 40, [mm.parallel(mm.attention(1, 1, 8, 8), space)])
    bits = mm.without(mm.weights(cfg, 11, memory=4.0), "left.o")
    ids = mm.tokens(cfg, 12, 150)
    m, e = make(cfg, bits, dtype)
    want = reference(cfg, bits, ids)
    assert mm.error(whole(m, e, ids), want) < TOL[dtype]
    assert mm.error(in_portions(m, e, ids, [65, 2, 17, 1, 5]), want) < TOL[dtype]
    assert mm.error(in_portions(m, e, ids[:40], [1]), want[:40]) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("layer", [mm.delta(1, 1, 8, 8, conv=1), mm.delta(6, 2, 40, 20, conv=2), mm.delta(4, 4, 64, 96), mm.delta(4, 1, 128, 33, conv=7),
                                   mm.delta(2, 2, 256, 256), mm.delta(3, 3, 65, 7), mm.delta(2, 1, 160, 70), mm.delta(2, 1, 224, 40)])
def test_delta_rule_alone(make, dtype, layer):
    cfg = mm.config(64, 40, [layer])
    bits = mm.weights(cfg, 13, memory=4.0)
    ids = mm.tokens(cfg, 14, 150)
    m, e = make(cfg, bits, dtype)
    want = reference(cfg, bits, ids)
    assert mm.error(whole(m, e, ids), want) < TOL[dtype]
    assert mm.error(in_portions(m, e, ids, [65, 2, 17, 1, 5]), want) < TOL[dtype]
    assert mm.error(in_portions(m, e, ids[:40], [1]), want[:40]) < TOL[dtype]


@pytest.mark.parametrize("a_log,dt_bias", [(-9.0, -3.0), (-3.0, 0.0), (0.0, 3.0), (3.0, 2.0), (4.0, -4.0), (5.0, 5.0)])
@pytest.mark.parametrize("kind", ["delta", "space"])
def test_decays_of_every_strength(make, kind, a_log, dt_bias):
    """From a state that hardly decays over the whole prompt to one that is gone within a token, mixed over the heads."""
    layer = mm.delta(4, 2, 24, 16) if kind == "delta" else mm.parallel(mm.attention(1, 1, 8, 8), mm.space(4, 16, 24))
    cfg = mm.config(64, 40, [layer])
    bits = mm.without(mm.weights(cfg, 15), "left.o")
    p = "l0.mix." if kind == "delta" else "l0.mix.right."
    bits[p + "A_log"] = mm.bf16_bits([a_log, a_log - 1.0, -6.0, a_log])
    bits[p + "dt_bias"] = mm.bf16_bits([dt_bias, dt_bias, 0.0, -dt_bias])
    ids = mm.tokens(cfg, 16, 200)
    m, e = make(cfg, bits)
    want = reference(cfg, bits, ids)
    assert mm.error(whole(m, e, ids), want) < TOL["float32"]
    assert mm.error(in_portions(m, e, ids, [70, 3, 1]), want) < TOL["float32"]


def test_repeated_keys(make):
    """The same token over and over: the delta rule's triangular system is as far from the identity as it gets."""
    cfg = mm.config(64, 40, [mm.delta(3, 1, 24, 32), mm.delta(2, 2, 48, 16)])
    bits = mm.weights(cfg, 17, memory=50.0)
    for i in range(2):
        bits = mm.scaled(bits, f"l{i}.mix.b", 6.0)   # (betas near 0 and 1)
    ids = [5] * 90 + [9] * 60 + mm.tokens(cfg, 18, 50) + [5] * 40
    m, e = make(cfg, bits)
    want = reference(cfg, bits, ids)
    assert mm.error(whole(m, e, ids), want) < TOL["float32"]
    assert mm.error(in_portions(m, e, ids, [100, 2, 1, 31]), want) < TOL["float32"]


# --- prompts, portions, decoding -------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,n", [("MIXED", 150), ("PLAIN", 200), ("WIDE", 140)])
def test_prompt_portions_and_decoding(make, dtype, name, n):
    cfg = getattr(mm, name)
    bits = mm.weights(cfg, 21)
    ids = mm.tokens(cfg, 22, n)
    m, e = make(cfg, bits, dtype)
    want = reference(cfg, bits, ids)
    assert mm.error(whole(m, e, ids), want) < TOL[dtype]
    for sizes in ([2], [3, 17], [16, 33, 1], [64, 2, 5], [n - 7, 1], [63, 66]):
        assert mm.error(in_portions(m, e, ids, sizes), want) < TOL[dtype], sizes
    assert mm.error(in_portions(m, e, ids, [1]), want) < TOL[dtype]
    assert m.uses_graph()


@pytest.mark.parametrize("n", [1, 2, 3, 15, 16, 17, 31, 32, 33, 63, 64, 65, 79, 80, 81, 127, 128, 129, 192, 193])
def test_prompt_lengths_at_tile_and_chunk_edges(make, n):
    """Then two more tokens, so that what the prompt leaves behind is looked at too."""
    cfg = mm.MIXED
    bits = mm.weights(cfg, 23)
    ids = mm.tokens(cfg, 24, n + 5)
    m, e = make(cfg, bits)
    want = reference(cfg, bits, ids)
    assert mm.error(whole(m, e, ids[:n]), want[:n]) < TOL["float32"]
    assert mm.error(in_portions(m, e, ids, [1, 2], at=n), want[n:]) < TOL["float32"]


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_prompts_in_segments(make, dtype):
    """More tokens than a chunked pass takes at a time, with states that remember all of them; then long decoding."""
    cfg = mm.config(48, 40, [mm.delta(2, 1, 16, 16), mm.parallel(mm.attention(1, 1, 8, 8), mm.space(2, 16, 16))])
    bits = mm.without(mm.weights(cfg, 25, memory=3000.0), "left.o")
    ids = mm.tokens(cfg, 26, 2300)
    m, e = make(cfg, bits, dtype, max_seq=2304)
    want = reference(cfg, bits, ids)
    tol = 1e-4 if dtype == "float32" else 0.1
    assert mm.error(whole(m, e, ids), want) < tol
    assert mm.error(in_portions(m, e, ids, [2050, 2, 40]), want) < tol
    got = [whole(m, e, ids[:2000])] + [m.forward_tokens(e, [t], 2000 + i) for i, t in enumerate(ids[2000:])]
    assert mm.error(np.concatenate(got), want) < tol


class Forgetful(plain.Sequence):
    """The oracle with one position's key and value taken out of every later token's history, or with every recurrent state
    set to zero behind it."""

    def __init__(self, cfg, w, lost, what):
        super().__init__(cfg, w)
        self.lost, self.what = lost, what

    def token(self, tok):
        out = super().token(tok)
        if self.position == self.lost + 1:
            for memory in self.memory:
                if self.what == "key" and "kv" in memory:
                    k, v = memory["kv"][self.lost]
                    memory["kv"][self.lost] = (np.zeros_like(k), np.zeros_like(v))
                if self.what == "state" and "s" in memory:
                    memory["s"][:] = 0
        return out


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("page", [0, 16, 64])
def test_far_keys_and_page_borders(make, dtype, page):
    """Queries sharp enough that a few single keys carry each output.  Every key of a long context counts: the oracle without
    one of them (the first tokens, both sides of page and chunk borders) differs by far more than the tolerance."""
    cfg = mm.config(64, 60, [mm.parallel(mm.attention(4, 2, 32, 24, scale=0.9), mm.space(1, 8, 8), left_scale=1.5),
                             mm.parallel(mm.attention(2, 2, 24, 24, scale=0.9), mm.space(1, 8, 8), left_scale=1.5)])
    bits = mm.without(mm.weights(cfg, 31, sink=0.3), "right.o")
    n = 290
    ids = mm.tokens(cfg, 32, n)
    w = mm.values(bits)
    want = plain.run(cfg, w, ids).logits
    m, e = make(cfg, bits, dtype, max_seq=320)
    if page:
        m.set_attention(page_size=page, n_pages=320 // page)
    tol = 1e-4 if dtype == "float32" else 0.2
    assert mm.error(whole(m, e, ids), want) < tol
    assert mm.error(in_portions(m, e, ids, [100, 2, 7, 31]), want) < tol
    got = np.concatenate([whole(m, e, ids[:250])] + [m.forward_tokens(e, [t], 250 + i) for i, t in enumerate(ids[250:])])
    assert mm.error(got, want) < tol
    if dtype == "float32" and page == 16:
        for lost in (0, 1, 15, 16, 63, 64, 127, 128, 200):
            seq = Forgetful(cfg, w, lost, "key")
            assert mm.error(seq.step(ids)[lost + 1:], want[lost + 1:]) > 50 * tol, lost


def test_states_remember_across_borders(make):
    """States that hardly decay: the oracle that loses them at a chunk's, a portion's or a decode step's border differs."""
    cfg = mm.config(64, 60, [mm.delta(2, 1, 24, 24), mm.parallel(mm.attention(1, 1, 8, 8), mm.space(2, 24, 24))])
    bits = mm.without(mm.weights(cfg, 33, memory=100.0), "left.o")
    ids = mm.tokens(cfg, 34, 200)
    w = mm.values(bits)
    want = plain.run(cfg, w, ids).logits
    m, e = make(cfg, bits)
    for sizes in ([200], [64, 64, 72], [100, 16, 1, 83], [150, 1]):
        assert mm.error(in_portions(m, e, ids, sizes), want) < TOL["float32"], sizes
    for lost in (63, 64, 99, 116, 150):
        assert mm.error(Forgetful(cfg, w, lost, "state").step(ids)[lost + 1:], want[lost + 1:]) > 100 * TOL["float32"], lost


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("slots", [1, 3])
def test_long_walks_of_the_decode_attention(make, monkeypatch, dtype, slots):
    """Few splits, so that each walks many chunks of keys through its ring of buffers: lone rows and portions, rows of several
    lengths, more heads than a tile."""
    monkeypatch.setenv("OXB_HIP_ATTN_SLOTS", str(slots))
    for a in (mm.attention(4, 2, 128, 128, scale=0.5), mm.attention(3, 1, 24, 200, scale=0.8), mm.attention(20, 1, 256, 40, scale=0.3), mm.attention(2, 1, 32, 16, scale=0.8)):
        cfg = mm.config(64, 50, [mm.parallel(a, mm.space(1, 8, 8))])
        bits = mm.without(mm.weights(cfg, 17), "right.o")
        ids = mm.tokens(cfg, 18, 330)
        m, e = make(cfg, bits, dtype, max_seq=384)
        want = reference(cfg, bits, ids)
        m.forward_tokens(e, ids[:250], 0, want=[])
        got = np.concatenate([m.forward_tokens(e, ids[at:at + k], at, want=range(k)) for at, k in ((250, 16), (266, 8), (274, 2), (276, 16))] +
                             [m.forward_tokens(e, [t], 292 + i) for i, t in enumerate(ids[292:])])
        assert mm.error(got, want[250:]) < (5e-5 if dtype == "float32" else 0.12)


def test_logits_of_chosen_tokens(make):
    cfg = mm.MIXED
    bits = mm.weights(cfg, 25)
    ids = mm.tokens(cfg, 26, 60)
    m, e = make(cfg, bits)
    want = reference(cfg, bits, ids)
    for pick in ([0], [59, 3, 3], [], list(range(20, 60))):
        got = m.forward_tokens(e, ids, 0, want=pick)
        assert got.shape == (len(pick), cfg["vocab"])
        if pick:
            assert mm.error(got, want[pick]) < TOL["float32"]
    logits, token = m.prefill_tokens(e, ids)
    assert mm.error(logits[None], want[-1:]) < TOL["float32"] and token == int(np.argmax(want[-1]))
    rows = mm.values(bits)["embed"]
    logits, token = m.prefill(rows[ids])
    assert mm.error(logits[None], want[-1:]) < TOL["float32"]
    got, tok = m.forward(rows[[7]], 60)
    assert mm.error(got, reference(cfg, bits, ids + [7])[-1:]) < TOL["float32"] and tok[0] == int(np.argmax(got[0]))


@pytest.mark.parametrize("dtype", DTYPES)
def test_batch_of_unequal_requests(make, dtype):
    """Three slots at different positions decode together; each gives what it gives alone."""
    cfg = mm.MIXED
    bits = mm.weights(cfg, 41)
    prompts = [mm.tokens(cfg, 42, 5), mm.tokens(cfg, 43, 90), mm.tokens(cfg, 44, 33)]
    tails = [mm.tokens(cfg, 45 + b, 12) for b in range(3)]
    w = mm.values(bits)
    want = [plain.run(cfg, w, p + t).logits for p, t in zip(prompts, tails)]
    for paged in (False, True):
        m, e = make(cfg, bits, dtype, batch=3)
        if paged:
            m.set_attention(page_size=16, n_pages=14)
        for b in (1, 0, 2):
            assert mm.error(whole(m, e, prompts[b], b), want[b][:len(prompts[b])]) < TOL[dtype]
        for i in range(12):
            rows = w["embed"][[t[i] for t in tails]]
            pos = [len(p) + i for p in prompts]
            logits, toks = m.forward(rows, pos)
            for b in range(3):
                assert mm.error(logits[b][None], want[b][pos[b]][None]) < TOL[dtype], (paged, i, b)
                assert toks[b] == int(np.argmax(logits[b]))
        # one slot goes on alone with a single token, then with a portion, while the others rest
        more = [3] + mm.tokens(cfg, 49, 20)
        at = len(prompts[1]) + 12
        got = np.concatenate([m.forward_tokens(e, more[:1], at, 1), m.forward_tokens(e, more[1:], at + 1, 1, want=range(20))])
        assert mm.error(got, plain.run(cfg, w, prompts[1] + tails[1] + more).logits[at:]) < TOL[dtype]


@pytest.mark.parametrize("B", [17, 70])
def test_large_batch(make, B):
    """More sequences than one column tile: the products go through the GEMM, attention and recurrences stay the decode form."""
    cfg = mm.config(64, 50, [mm.delta(2, 1, 16, 24, ff=80), mm.parallel(mm.attention(2, 1, 16, 24), mm.space(2, 16, 16), ff=80)])
    bits = mm.weights(cfg, 51)
    prompts = [mm.tokens(cfg, 60 + b, 3 + (2 * b) % 23) for b in range(B)]
    m, e = make(cfg, bits, batch=B, max_seq=64)
    for b in range(B):
        m.forward_tokens(e, prompts[b], 0, b, want=[])
    nxt = mm.tokens(cfg, 52, B)
    logits, _ = m.forward(mm.values(bits)["embed"][nxt], [len(p) for p in prompts])
    for b in (0, 7, 15, 16, B - 1):
        assert mm.error(logits[b][None], reference(cfg, bits, prompts[b] + [nxt[b]])[-1:]) < TOL["float32"], b


def test_pages_and_slots_are_reused(make):
    """Released pages and slots come back under another request; nothing of the old one shows."""
    cfg = mm.MIXED
    bits = mm.weights(cfg, 61, memory=50.0)
    m, e = make(cfg, bits, batch=2, max_seq=128)
    m.set_attention(page_size=16, n_pages=9)
    a, b, c = mm.tokens(cfg, 62, 60), mm.tokens(cfg, 63, 70), mm.tokens(cfg, 64, 100)
    assert mm.error(in_portions(m, e, a, [20, 2], 0), reference(cfg, bits, a)) < TOL["float32"]
    assert mm.error(in_portions(m, e, b, [33, 5], 1), reference(cfg, bits, b)) < TOL["float32"]
    assert m.kv_pool().free_pages == 0
    m.kv_release(0)
    assert m.kv_pool().free_pages == 4
    b2 = b + mm.tokens(cfg, 65, 20)   # the living request grows into the other's pages
    got = m.forward_tokens(e, b2[70:], 70, 1, want=range(20))
    assert mm.error(got, reference(cfg, bits, b2)[70:]) < TOL["float32"]
    m.kv_release(1)
    for first in (2, 40, 1):   # a new request's first portion in every form: steps, chunks, one token
        assert mm.error(in_portions(m, e, c, [first, 40, 1], 0), reference(cfg, bits, c)) < TOL["float32"]
        m.kv_release(0)
    m.reset()
    assert m.kv_pool().free_pages == 9
    # a contiguous slot used again without a word: position 0 starts a new request
    m.set_attention()
    whole(m, e, c, 1)
    assert mm.error(in_portions(m, e, a[:9], [1], 1), reference(cfg, bits, a[:9])) < TOL["float32"]
    assert mm.error(in_portions(m, e, a[:9], [4, 1], 1), reference(cfg, bits, a[:9])) < TOL["float32"]
    with pytest.raises(Exception):
        m.set_attention(1)
    with pytest.raises(Exception):
        m.set_attention(0, window_size=16)


def test_states_go_on_where_they_stand(make):
    """A recurrent state cannot be wound back: portions and steps elsewhere are refused, and change nothing."""
    from oxibonsai_amd.backend import GpuError
    cfg = mm.PLAIN
    bits = mm.weights(cfg, 66)
    ids = mm.tokens(cfg, 67, 40)
    m, e = make(cfg, bits, batch=2)
    want = reference(cfg, bits, ids)
    m.forward_tokens(e, ids[:30], 0, 0, want=[])
    m.forward_tokens(e, ids[:20], 0, 1, want=[])
    for pos in (29, 31, 5):
        with pytest.raises(GpuError, match="stands at position 30"):
            m.forward_tokens(e, ids[30:32], pos, 0)
    with pytest.raises(GpuError, match="stands at position 20"):
        m.forward(mm.values(bits)["embed"][[1, 1]], [30, 19])
    with pytest.raises(GpuError, match="stands at position 30"):
        m.generate(e, [1, 1], [31, 20], 2)
    assert mm.error(in_portions(m, e, ids, [3], 0, at=30), want[30:]) < TOL["float32"]
    assert mm.error(in_portions(m, e, ids, [17, 1], 1, at=20), want[20:]) < TOL["float32"]
    m.kv_release(0)
    with pytest.raises(GpuError, match="stands at position 0"):
        m.forward_tokens(e, ids[:2], 40, 0)


def test_sizes_beyond_the_kernels_are_refused(backend):
    from oxibonsai_amd.backend import GpuError
    from oxibonsai_amd.model import HipModel
    for layer, says in ((mm.delta(1, 1, 300, 8), "beyond 256"), (mm.parallel(mm.attention(1, 1, 300, 8), mm.space(1, 8, 8)), "beyond 256")):
        cfg = mm.config(16, 10, [layer])
        with pytest.raises(GpuError, match=says):
            HipModel.from_tensors(backend, cfg, mm.weights(cfg, 1))
    bits = mm.weights(mm.PLAIN, 1)
    for name in ("l0.mix.right.conv", "l1.mix.A_log", "l0.mlp.up", "final.norm"):
        with pytest.raises(GpuError, match=name):
            HipModel.from_tensors(backend, mm.PLAIN, {k: (v[:-1] if k == name else v) for k, v in bits.items()})
        with pytest.raises(GpuError, match=name):
            HipModel.from_tensors(backend, mm.PLAIN, {k: v for k, v in bits.items() if k != name})


def test_results_do_not_depend_on_the_cut_beyond_rounding(make):
    """bf16: every cut lies as close to every other as to the exact result."""
    cfg = mm.PLAIN
    bits = mm.weights(cfg, 71)
    ids = mm.tokens(cfg, 72, 120)
    m, e = make(cfg, bits, "bfloat16")
    runs = [whole(m, e, ids)] + [in_portions(m, e, ids, s) for s in ([1], [2], [50, 3], [17])]
    for r in runs[1:]:
        assert mm.error(r, runs[0]) < TOL["bfloat16"]


# --- generation ------------------------------------------------------------------------------------------------------
def check_greedy(cfg, w, prompt, ids, tol):
    """Every generated token is the oracle's argmax given the tokens before it, up to ties within rounding."""
    logits = plain.run(cfg, w, prompt + list(ids[:-1])).logits[len(prompt) - 1:]
    for i, t in enumerate(ids):
        assert logits[i].max() - logits[i][t] <= tol * np.std(logits[i]), i


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation(make, dtype):
    """Prompts of two slots, then the token loop on the device, long enough to cross chunks of the decode attention."""
    cfg = mm.config(64, 100, [mm.delta(2, 1, 16, 24, ff=80), mm.parallel(mm.attention(3, 1, 16, 16), mm.space(2, 16, 16), ff=80)])
    bits = mm.weights(cfg, 81)
    w = mm.values(bits)
    prompts = [mm.tokens(cfg, 82, 30), mm.tokens(cfg, 83, 7)]
    m, e = make(cfg, bits, dtype, batch=2)
    first = [m.prefill_tokens(e, p, 0, b)[1] for b, p in enumerate(prompts)]
    n = 140
    ids = m.generate(e, first, [len(p) for p in prompts], n)
    for b in range(2):
        check_greedy(cfg, w, prompts[b], [first[b]] + [int(t) for t in ids[:, b]], 1e-4 if dtype == "float32" else 0.25)
    # in two calls: the states go on
    first = [m.prefill_tokens(e, p, 0, b)[1] for b, p in enumerate(prompts)]
    a = m.generate(e, first, [len(p) for p in prompts], 9)
    b = m.generate(e, a[-1], [len(p) + 9 for p in prompts], 11)
    assert np.array_equal(np.concatenate([a, b]), ids[:20])
    # sampled: temperature near zero is greedy, a real temperature gives tokens of the vocabulary and moves the generator
    first = [m.prefill_tokens(e, p, 0, b)[1] for b, p in enumerate(prompts)]
    cold, _ = m.generate_sampled(e, first, [len(p) for p in prompts], 20, 1e-7, 40, 0.9, [1, 2])
    assert np.array_equal(cold, ids[:20])
    first = [m.prefill_tokens(e, p, 0, b)[1] for b, p in enumerate(prompts)]
    warm, rng = m.generate_sampled(e, first, [len(p) for p in prompts], 20, 1.0, 40, 0.9, [1, 2])
    assert warm.max() < cfg["vocab"] and not np.array_equal(rng, [1, 2])


def test_checkpoint_folder_and_command_line(tmp_path, backend):
    """The same model from a folder: loader, info, `python -m oxibonsai_amd generate`, and the trace runner, whose requests
    take turns in one slot."""
    from oxibonsai_amd.model import HipModel
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = mm.MIXED
    bits = mm.weights(cfg, 91)
    path = mm.write_checkpoint(tmp_path, cfg, bits)
    ids = mm.tokens(cfg, 92, 40)
    want = reference(cfg, bits, ids)
    m, e, info = HipModel.from_checkpoint(backend, path, "float32", max_seq=128)
    assert info["architecture"] == "Muvonex" and info["n_layers"] == 4 and info["vocab"] == cfg["vocab"]
    assert mm.error(whole(m, e, ids), want) < TOL["float32"]
    m.close()
    e.close()
    env = dict(os.environ, PYTHONPATH=root)
    r = subprocess.run([sys.executable, "-m", "oxibonsai_amd", "generate", path, "--dtype", "float32", "--tokens", ",".join(map(str, ids)),
                        "--steps", "12", "--max-seq", "128"], capture_output=True, text=True, env=env, timeout=100)
    assert r.returncode == 0, r.stderr
    check_greedy(cfg, mm.values(bits), ids, [int(t) for t in r.stdout.split()], 1e-4)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": ids[:25], "want": [0, 24]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": ids[25:27], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": [ids[27]], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": ids[:1], "want": [0]}], "end": []},
             {"step": 4, "entries": [{"id": "b", "tokens": ids[1:9], "want": [7]}], "end": ["b"]}]
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "28"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, env=env, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(5)]
    for step, rows in ((0, [0, 24]), (2, [27]), (3, [0]), (4, [8])):
        got = np.fromfile(tmp_path / f"{step}.f32", "<f4").reshape(-1, cfg["vocab"])
        assert mm.error(got, want[rows]) < TOL["float32"]
    assert not (tmp_path / "1.f32").exists()
