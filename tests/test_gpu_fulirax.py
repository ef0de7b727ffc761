"""Fulirax on the GPU against its plain oracle (oracle/plain_fulirax.py): mechanisms alone, prompts, portions, decoding,
batches, pages, greedy generation; fp32 within rounding of 32 bits, bf16 within rounding of its products."""
from __future__ import annotations

import json
import subprocess
import sys

import numpy as np
import pytest

import fulirax_models as fm
from oracle import plain_fulirax as plain

pytestmark = pytest.mark.gpu

TOL = {"float32": 2e-5, "bfloat16": 6e-2}
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
    return plain.run(cfg, fm.values(bits), ids).logits


def whole(m, e, ids, seq=0):
    return m.forward_tokens(e, ids, 0, seq, want=range(len(ids)))


def in_portions(m, e, ids, sizes, seq=0):
    """The prompt cut into portions of the given sizes, cyclically."""
    out, at, k = [], 0, 0
    while at < len(ids):
        n = min(sizes[k % len(sizes)], len(ids) - at)
        out.append(m.forward_tokens(e, ids[at:at + n], at, seq, want=range(n)))
        at, k = at + n, k + 1
    return np.concatenate(out)


# --- mechanisms alone: everything else is switched off through the weights -------------------------------------------
def without_attention(bits):
    return {k: (np.zeros_like(v) if k.endswith("mix.o") else v) for k, v in bits.items()}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("alpha", [1e-3, 0.05, 0.7, 6.0])
def test_dynamic_tanh_alone(make, dtype, alpha):
    cfg = fm.config(90, 77, [fm.layer(1, 8, 4, 8, 16)])
    bits = without_attention(fm.weights(cfg, 1))
    bits["final.norm.alpha"] = fm.bf16_bits(alpha)
    if alpha < 0.01:
        bits["final.norm"] = fm.bf16_bits(fm.bf16_value(bits["final.norm"]) * 300.0)   # tanh near zero, magnified
    ids = fm.tokens(cfg, 2, 40)
    m, e = make(cfg, bits, dtype)
    w = fm.values(bits)
    x = w["embed"][ids].astype(np.float64)
    want = plain.norm(x, "final.norm", {k: v.astype(np.float64) for k, v in w.items()}) @ w["embed"].T.astype(np.float64) * cfg["logit_scale"]
    assert fm.error(whole(m, e, ids), want) < (2e-6 if dtype == "float32" else 1e-2)
    assert fm.error(reference(cfg, bits, ids[:5]), want[:5]) < 1e-12


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("gain", [0.02, 1.0, 8.0])
def test_feed_forward_alone(make, dtype, gain):
    cfg = fm.config(72, 50, [fm.layer(1, 8, 4, 8, 16, ff=133)])
    bits = without_attention(fm.weights(cfg, 3))
    bits["l0.mlp.up"] = fm.bf16_bits(fm.bf16_value(bits["l0.mlp.up"]) * gain)
    bits["l0.mlp.down"] = fm.bf16_bits(fm.bf16_value(bits["l0.mlp.down"]) * (2.0 / gain))
    ids = fm.tokens(cfg, 4, 24)
    m, e = make(cfg, bits, dtype)
    assert fm.error(whole(m, e, ids), reference(cfg, bits, ids)) < (5e-6 if dtype == "float32" else 2e-2)


@pytest.mark.parametrize("times", [1, 3])
def test_loop_entry_alone(make, times):
    cfg = fm.config(66, 40, [fm.layer(1, 8, 4, 8, 16), fm.layer(1, 8, 4, 8, 16)], loop=(1, 2, times))
    bits = without_attention(fm.weights(cfg, 5))
    ids = fm.tokens(cfg, 6, 20)
    m, e = make(cfg, bits)
    want = reference(cfg, bits, ids)
    assert fm.error(whole(m, e, ids), want) < 5e-6
    # the pass's vector and the embedding output both matter
    for name in ("loop.step", "loop.in"):
        other = dict(bits)
        a = fm.bf16_value(bits[name]).copy()
        if name == "loop.step":
            a[-1] = 0
        else:
            a[:, cfg["width"]:] = 0
        other[name] = fm.bf16_bits(a)
        assert fm.error(reference(cfg, other, ids), want) > 1e-2


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sink", [-40.0, 0.0, 4.0, 30.0])
@pytest.mark.parametrize("n", [1, 3, 40])
def test_sink(make, dtype, sink, n):
    """From a sink that takes nothing to one that takes everything; decided alone (n = 1), in a short portion, in a prompt."""
    cfg = fm.config(64, 40, [fm.layer(3, 16, 8, 24, 32)])
    bits = fm.weights(cfg, 7)
    bits["l0.mix.sink"] = fm.bf16_bits([sink, sink + 1.0, sink - 2.0])
    ids = fm.tokens(cfg, 8, n)
    m, e = make(cfg, bits, dtype)
    want = reference(cfg, bits, ids)
    assert fm.error(whole(m, e, ids), want) < TOL[dtype]
    assert fm.error(in_portions(m, e, ids, [1]), want) < TOL[dtype]


def test_rotation_base_and_partial_rotation(make):
    """Positions matter through the rotated part alone, with a base per layer and rotated dimensions that may be fewer than
    the part's."""
    cfg = fm.config(80, 30, [fm.layer(2, 16, 24, 16, 40, base=30.0, rot_dims=10, scale=0.6), fm.layer(2, 16, 10, 16, 40, base=1e6, scale=0.6)])
    bits = fm.weights(cfg, 9)
    ids = [3] * 4 + fm.tokens(cfg, 10, 150)
    m, e = make(cfg, bits)
    want = reference(cfg, bits, ids)
    assert fm.error(whole(m, e, ids), want) < TOL["float32"]
    cfg2 = json.loads(json.dumps(cfg))
    cfg2["layers"][0]["mixer"]["rot"]["base"] = 33.0
    assert fm.error(reference(cfg2, bits, ids), want) > 1e-2


def test_latent_norm_eps(make):
    """Small latents, so that eps decides."""
    cfg = fm.config(64, 40, [fm.layer(2, 16, 8, 24, 48)], eps=0.03)
    bits = fm.weights(cfg, 11)
    bits["l0.mix.dkv"] = fm.bf16_bits(fm.bf16_value(bits["l0.mix.dkv"]) * 0.1)
    ids = fm.tokens(cfg, 12, 30)
    m, e = make(cfg, bits)
    want = reference(cfg, bits, ids)
    assert fm.error(whole(m, e, ids), want) < TOL["float32"]
    assert fm.error(reference(dict(cfg, norm={"eps": 1e-5}), bits, ids), want) > 1e-2


# --- prompts, portions, decoding -------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,n", [("MIXED", 150), ("PLAIN", 200), ("ONCE", 70), ("WIDE", 50)])
def test_prompt_portions_and_decoding(make, dtype, name, n):
    cfg = getattr(fm, name)
    bits = fm.weights(cfg, 21)
    ids = fm.tokens(cfg, 22, n)
    m, e = make(cfg, bits, dtype)
    want = reference(cfg, bits, ids)
    assert fm.error(whole(m, e, ids), want) < TOL[dtype]
    for sizes in ([2], [3, 17], [16, 33, 1], [64, 2, 5], [n - 7, 1]):
        assert fm.error(in_portions(m, e, ids, sizes), want) < TOL[dtype], sizes
    assert fm.error(in_portions(m, e, ids, [1]), want) < TOL[dtype]
    assert m.uses_graph()


@pytest.mark.parametrize("n", [1, 2, 15, 16, 17, 31, 32, 33, 63, 64, 65, 127, 128, 129])
def test_prompt_lengths_at_tile_edges(make, n):
    cfg = fm.PLAIN
    bits = fm.weights(cfg, 23)
    ids = fm.tokens(cfg, 24, n)
    m, e = make(cfg, bits)
    assert fm.error(whole(m, e, ids), reference(cfg, bits, ids)) < TOL["float32"]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff,n", [(3072, 512), (3072, 700), (3072, 1950), (2112, 1800), (520, 300), (3072, 40)])
def test_products_at_every_tile_size(make, dtype, ff, n):
    """Feed-forward alone at widths and prompt lengths that take the GEMM through its tile sizes, last tiles ragged."""
    cfg = fm.config(200, 64, [fm.layer(1, 8, 4, 8, 16, ff=ff)])
    bits = without_attention(fm.weights(cfg, 13))
    ids = fm.tokens(cfg, 14, n)
    m, e = make(cfg, bits, dtype, max_seq=2048)
    w = {k: v.astype(np.float64) for k, v in fm.values(bits).items()}
    x = w["embed"][ids]
    x = x + plain.gelu_tanh(plain.norm(x, "l0.norm2", w) @ w["l0.mlp.up"].T) @ w["l0.mlp.down"].T
    want = plain.norm(x, "final.norm", w) @ w["embed"].T * cfg["logit_scale"]
    assert fm.error(whole(m, e, ids), want) < (5e-6 if dtype == "float32" else 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,rot,vdim,rank,n", [(24, 128, 64, 128, 512, 420), (16, 96, 32, 64, 256, 300), (9, 192, 64, 200, 130, 200)])
def test_large_heads(make, dtype, heads, dim, rot, vdim, rank, n):
    """Head and latent sizes of large models: prompt, short portions, decoding behind a long context."""
    cfg = fm.config(192, 80, [fm.layer(heads, dim, rot, vdim, rank)])
    bits = fm.weights(cfg, 15, sharp=1.5)
    ids = fm.tokens(cfg, 16, n)
    m, e = make(cfg, bits, dtype, max_seq=512)
    want = plain.run_prompt(cfg, fm.values(bits), ids)
    assert fm.error(whole(m, e, ids), want) < TOL[dtype]
    got = np.concatenate([in_portions(m, e, ids[:n - 60], [150, 90])] +
                         [m.forward_tokens(e, ids[at:at + k], at, want=range(k)) for at, k in ((n - 60, 16), (n - 44, 9), (n - 35, 3))] +
                         [m.forward_tokens(e, [t], n - 32 + i) for i, t in enumerate(ids[n - 32:])])
    assert fm.error(got, want) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("slots", [1, 3])
def test_long_walks_of_the_decode_attention(make, monkeypatch, dtype, slots):
    """Few splits, so that each walks many chunks of keys through its ring of buffers: lone rows and portions, one head tile
    and two, latent sizes with rings of four buffers down to one."""
    monkeypatch.setenv("OXB_HIP_ATTN_SLOTS", str(slots))
    for layers in ([fm.layer(18, 32, 16, 24, 64, scale=0.4), fm.layer(3, 24, 8, 16, 300)], [fm.layer(2, 16, 8, 16, 640), fm.layer(20, 16, 8, 8, 500)]):
        cfg = fm.config(64, 50, layers)
        bits = fm.weights(cfg, 17, sharp=2.0)
        ids = fm.tokens(cfg, 18, 330)
        m, e = make(cfg, bits, dtype, max_seq=384)
        want = plain.run_prompt(cfg, fm.values(bits), ids)
        m.forward_tokens(e, ids[:250], 0, want=[])
        got = np.concatenate([m.forward_tokens(e, ids[at:at + k], at, want=range(k)) for at, k in ((250, 16), (266, 8), (274, 2), (276, 16))] +
                             [m.forward_tokens(e, [t], 292 + i) for i, t in enumerate(ids[292:])])
        assert fm.error(got, want[250:]) < (5e-5 if dtype == "float32" else 0.12)


def test_logits_of_chosen_tokens(make):
    cfg = fm.MIXED
    bits = fm.weights(cfg, 25)
    ids = fm.tokens(cfg, 26, 60)
    m, e = make(cfg, bits)
    want = reference(cfg, bits, ids)
    for pick in ([0], [59, 3, 3], [], list(range(20, 60))):
        got = m.forward_tokens(e, ids, 0, want=pick)
        assert got.shape == (len(pick), cfg["vocab"])
        if pick:
            assert fm.error(got, want[pick]) < TOL["float32"]
    logits, token = m.prefill_tokens(e, ids)
    assert fm.error(logits[None], want[-1:]) < TOL["float32"] and token == int(np.argmax(want[-1]))
    rows = fm.values(bits)["embed"][ids]
    logits, token = m.prefill(rows)
    assert fm.error(logits[None], want[-1:]) < TOL["float32"]
    got, tok = m.forward(fm.values(bits)["embed"][[7]], 60)
    assert fm.error(got, reference(cfg, bits, ids + [7])[-1:]) < TOL["float32"] and tok[0] == int(np.argmax(got[0]))


def far_model(seed):
    """Queries sharp enough that a few single keys carry each output."""
    cfg = fm.config(64, 60, [fm.layer(2, 32, 16, 24, 64, scale=0.5), fm.layer(2, 24, 8, 24, 48, scale=0.5)])
    return cfg, fm.weights(cfg, seed, sharp=3.0, sink=0.3)


class Forgetful(plain.Sequence):
    """The oracle with one position's latent taken out of every later token's history."""

    def __init__(self, cfg, w, lost):
        super().__init__(cfg, w)
        self.lost = lost

    def token(self, tok):
        out = super().token(tok)
        if self.position == self.lost + 1:
            for h in self.history:
                c, r = h[self.lost]
                h[self.lost] = (np.zeros_like(c), np.zeros_like(r))
        return out


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("page", [0, 16, 64])
def test_far_keys_and_page_borders(make, dtype, page):
    """Every key of a long context counts: the oracle without one of them (the first tokens, both sides of page and chunk
    borders) differs by far more than the tolerance, the product does not."""
    cfg, bits = far_model(31)
    n = 290
    ids = fm.tokens(cfg, 32, n)
    w = fm.values(bits)
    want = plain.run(cfg, w, ids).logits
    m, e = make(cfg, bits, dtype, max_seq=320)
    if page:
        m.set_attention(page_size=page, n_pages=320 // page)
    tol = 1e-4 if dtype == "float32" else 0.2
    assert fm.error(whole(m, e, ids), want) < tol
    assert fm.error(in_portions(m, e, ids, [100, 2, 7, 31]), want) < tol
    got = np.concatenate([m.forward_tokens(e, ids[:250], 0, want=range(250))] + [m.forward_tokens(e, [t], 250 + i) for i, t in enumerate(ids[250:])])
    assert fm.error(got, want) < tol
    if dtype == "float32" and page == 16:
        for lost in (0, 1, 15, 16, 63, 64, 127, 128, 200):
            seq = Forgetful(cfg, w, lost)
            assert fm.error(seq.step(ids)[lost + 1:], want[lost + 1:]) > 50 * tol, lost


@pytest.mark.parametrize("dtype", DTYPES)
def test_batch_of_unequal_requests(make, dtype):
    """Three slots at different positions decode together; each gives what it gives alone."""
    cfg = fm.MIXED
    bits = fm.weights(cfg, 41)
    prompts = [fm.tokens(cfg, 42, 5), fm.tokens(cfg, 43, 90), fm.tokens(cfg, 44, 33)]
    tails = [fm.tokens(cfg, 45 + b, 12) for b in range(3)]
    w = fm.values(bits)
    want = [plain.run(cfg, w, p + t).logits for p, t in zip(prompts, tails)]
    for paged in (False, True):
        m, e = make(cfg, bits, dtype, batch=3)
        if paged:
            m.set_attention(page_size=16, n_pages=14)
        for b in (1, 0, 2):
            assert fm.error(whole(m, e, prompts[b], b), want[b][:len(prompts[b])]) < TOL[dtype]
        for i in range(12):
            rows = w["embed"][[t[i] for t in tails]]
            pos = [len(p) + i for p in prompts]
            logits, toks = m.forward(rows, pos)
            for b in range(3):
                assert fm.error(logits[b][None], want[b][pos[b]][None]) < TOL[dtype], (paged, i, b)
                assert toks[b] == int(np.argmax(logits[b]))
        # one slot goes on alone with a single token while the others rest
        got = m.forward_tokens(e, [3], len(prompts[1]) + 12, 1)
        assert fm.error(got, plain.run(cfg, w, prompts[1] + tails[1] + [3]).logits[-1:]) < TOL[dtype]


def test_large_batch(make):
    """More sequences than one column tile: the products go through the GEMM, attention stays the decode form."""
    cfg = fm.config(64, 50, [fm.layer(2, 16, 8, 24, 32, ff=80)])
    bits = fm.weights(cfg, 51)
    B = 21
    prompts = [fm.tokens(cfg, 60 + b, 3 + 2 * b) for b in range(B)]
    m, e = make(cfg, bits, batch=B, max_seq=64)
    for b in range(B):
        m.forward_tokens(e, prompts[b], 0, b, want=[])
    nxt = fm.tokens(cfg, 52, B)
    logits, _ = m.forward(fm.values(bits)["embed"][nxt], [len(p) for p in prompts])
    for b in (0, 7, 15, 16, 20):
        assert fm.error(logits[b][None], reference(cfg, bits, prompts[b] + [nxt[b]])[-1:]) < TOL["float32"], b


def test_pages_and_slots_are_reused(make):
    """Released pages come back in another order under another request; nothing of the old one shows."""
    cfg = fm.MIXED
    bits = fm.weights(cfg, 61)
    m, e = make(cfg, bits, batch=2, max_seq=128)
    m.set_attention(page_size=16, n_pages=9)
    a, b, c = fm.tokens(cfg, 62, 60), fm.tokens(cfg, 63, 70), fm.tokens(cfg, 64, 100)
    assert fm.error(in_portions(m, e, a, [20, 2], 0), reference(cfg, bits, a)) < TOL["float32"]
    assert fm.error(in_portions(m, e, b, [33, 5], 1), reference(cfg, bits, b)) < TOL["float32"]
    assert m.kv_pool().free_pages == 0
    m.kv_release(0)
    assert m.kv_pool().free_pages == 4
    b2 = b + fm.tokens(cfg, 65, 20)   # the living request grows into the other's pages
    got = m.forward_tokens(e, b2[70:], 70, 1, want=range(20))
    assert fm.error(got, reference(cfg, bits, b2)[70:]) < TOL["float32"]
    m.kv_release(1)
    assert fm.error(in_portions(m, e, c, [2, 40, 1], 0), reference(cfg, bits, c)) < TOL["float32"]
    m.reset()
    assert m.kv_pool().free_pages == 9
    # a contiguous slot used again: what lies behind the new request's end does not count
    m.set_attention()
    whole(m, e, c, 1)
    assert fm.error(in_portions(m, e, a[:9], [4, 1], 1), reference(cfg, bits, a[:9])) < TOL["float32"]
    with pytest.raises(Exception):
        m.set_attention(1)
    with pytest.raises(Exception):
        m.set_attention(0, window_size=16)


def test_results_do_not_depend_on_the_cut_beyond_rounding(make):
    """bf16: every cut lies as close to every other as to the exact result."""
    cfg = fm.ONCE
    bits = fm.weights(cfg, 71)
    ids = fm.tokens(cfg, 72, 120)
    m, e = make(cfg, bits, "bfloat16")
    runs = [whole(m, e, ids)] + [in_portions(m, e, ids, s) for s in ([1], [2], [50, 3], [17])]
    for r in runs[1:]:
        assert fm.error(r, runs[0]) < TOL["bfloat16"]


# --- generation ------------------------------------------------------------------------------------------------------
def check_greedy(cfg, w, prompt, ids, tol):
    """Every generated token is the oracle's argmax given the tokens before it, up to ties within rounding."""
    logits = plain.run(cfg, w, prompt + list(ids[:-1])).logits[len(prompt) - 1:]
    for i, t in enumerate(ids):
        assert logits[i].max() - logits[i][t] <= tol * np.std(logits[i]), i


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation(make, dtype):
    """Prompts of two slots, then the token loop on the device, long enough to cross chunks of the decode attention."""
    cfg = fm.config(64, 100, [fm.layer(2, 16, 8, 24, 32, ff=80), fm.layer(3, 16, 8, 16, 40, ff=80)], loop=(0, 1, 2))
    bits = fm.weights(cfg, 81)
    w = fm.values(bits)
    prompts = [fm.tokens(cfg, 82, 30), fm.tokens(cfg, 83, 7)]
    m, e = make(cfg, bits, dtype, batch=2)
    first = [m.prefill_tokens(e, p, 0, b)[1] for b, p in enumerate(prompts)]
    n = 140
    ids = m.generate(e, first, [len(p) for p in prompts], n)
    for b in range(2):
        check_greedy(cfg, w, prompts[b], [first[b]] + [int(t) for t in ids[:, b]], 1e-4 if dtype == "float32" else 0.25)
    # sampled: temperature near zero is greedy, a real temperature gives tokens of the vocabulary and moves the generator
    first = [m.prefill_tokens(e, p, 0, b)[1] for b, p in enumerate(prompts)]
    cold, _ = m.generate_sampled(e, first, [len(p) for p in prompts], 20, 1e-7, 40, 0.9, [1, 2])
    assert np.array_equal(cold, ids[:20])
    warm, rng = m.generate_sampled(e, first, [len(p) for p in prompts], 20, 1.0, 40, 0.9, [1, 2])
    assert warm.max() < cfg["vocab"] and not np.array_equal(rng, [1, 2])


def test_checkpoint_folder_and_command_line(tmp_path, backend):
    """The same model from a folder: loader, info, `python -m oxibonsai_amd generate`, and the trace runner."""
    import os
    from oxibonsai_amd.model import HipModel
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = fm.PLAIN
    bits = fm.weights(cfg, 91)
    path = fm.write_checkpoint(tmp_path, cfg, bits)
    ids = fm.tokens(cfg, 92, 40)
    want = reference(cfg, bits, ids)
    m, e, info = HipModel.from_checkpoint(backend, path, "float32", max_seq=128)
    assert info["architecture"] == "Fulirax" and info["n_layers"] == 2 and info["vocab"] == cfg["vocab"]
    assert fm.error(whole(m, e, ids), want) < TOL["float32"]
    m.close()
    e.close()
    env = dict(os.environ, PYTHONPATH=root)
    r = subprocess.run([sys.executable, "-m", "oxibonsai_amd", "generate", path, "--dtype", "float32", "--tokens", ",".join(map(str, ids)),
                        "--steps", "12", "--max-seq", "128"], capture_output=True, text=True, env=env, timeout=100)
    assert r.returncode == 0, r.stderr
    check_greedy(cfg, fm.values(bits), ids, [int(t) for t in r.stdout.split()], 1e-4)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": ids[:25], "want": [0, 24]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": ids[25:27], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": [ids[27]], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": ids[:9], "want": [8]}], "end": ["b"]}]
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "28"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, env=env, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    for step, rows in ((0, [0, 24]), (2, [27]), (3, [8])):
        got = np.fromfile(tmp_path / f"{step}.f32", "<f4").reshape(-1, cfg["vocab"])
        assert fm.error(got, want[rows]) < TOL["float32"]
    assert not (tmp_path / "1.f32").exists()
