"""Latent attention, norms behind sublayers, biased silu feed-forwards (Pabalix) on the GPU against the float64 oracle (oracle/stack_oracle.py)."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from oracle import stack_oracle as so
from stack_models import BF16_TOL, F32_TOL, bits, floats, gla, lat, lconfig, load, par, rel, tokens, weights

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {"float32": F32_TOL, "bfloat16": BF16_TOL}
YARN = (4.0, 64.0, 8.0, 1.0)             # factor, original, fast, slow
MIXED = [lat(2, rot=16, ff=48), lat(1, yarn=YARN), lat(3, heads=5, dim=24, vdim=12, kv_rank=40, yarn=YARN, ff=40), lat(2, heads=2, dim=40, rot=16, kv_from=0, ff=24)]


def whole(m, ids, want=None, stream=0, pos0=0):
    return m.step([(stream, ids, pos0, list(range(len(ids))) if want is None else want)])[0]


def by_token(m, ids, stream=0, pos0=0):
    rows = []
    for i, t in enumerate(ids):
        m.forward(t, pos0 + i, stream)
        rows.append(m.state.logits.copy())
    return np.array(rows)


def bound(dtype, cfg, fl, ids, want):
    """The tolerance, or what rounding the embedding alone does to a model that amplifies it."""
    bent = dict(fl)
    bent["embed"] = fl["embed"] * (1 + np.random.default_rng(0).uniform(-1, 1, fl["embed"].shape) * (2.0 ** -8 if dtype == "bfloat16" else 2.0 ** -23))
    return max(TOL[dtype], 8 * rel(so.forward(cfg, bent, ids), want))


# ---- every mechanism by itself: the residual stream behind every layer and the logits ------------------------------------------

def _no_mixer(w):
    w["l0.mix.o"] = np.zeros_like(w["l0.mix.o"])


ALONE = {
    "embedding_and_untied_head": (lconfig([lat()]), _no_mixer),
    "half_vector_pairs": (lconfig([lat(1, base=50.0)]), None),
    "half_vector_pairs_with_yarn": (lconfig([lat(1, rot=16, base=50.0, yarn=YARN)]), None),
    "adjacent_pairs": (lconfig([lat(2, base=50.0)]), None),
    "sink_and_head_gate": (lconfig([lat(3)]), None),
    "sink_gate_and_yarn": (lconfig([lat(3, rot=12, yarn=(2.5, 40.0, 6.0, 0.5))]), None),
    "latents_of_an_earlier_layer": (lconfig([lat(2), lat(1), lat(2, kv_from=0), lat(2, heads=2, kv_from=0)]), None),
    "feed_forward": (lconfig([lat(ff=72)]), _no_mixer),
    "eps_that_matters": (lconfig([lat(2, ff=24)], eps=0.3), None),
    "all_kinds": (lconfig(MIXED), None),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(ALONE))
def test_mechanism_alone(name, dtype):
    cfg, edit = ALONE[name]
    w = weights(cfg, 3)
    if edit:
        edit(w)
    ids = tokens(70, seed=5)
    fl = floats(w)
    want, layers = so.forward(cfg, fl, ids, want_layers=True)
    tol = bound(dtype, cfg, fl, ids, want)
    m = load(cfg, w, dtype)
    m.trace_layers(True)
    got = whole(m, ids)
    seen = m.layer_trace(len(ids))
    m.trace_layers(False)
    assert seen.shape == layers.shape
    for r in range(len(layers)):
        assert rel(seen[r], layers[r]) < tol, r
    assert rel(got, want) < tol
    assert rel(by_token(m, ids, stream=1), want) < tol
    m.close()


# ---- sizes ----------------------------------------------------------------------------------------------------------------------

SIZES = {
    "odd": lconfig([lat(2, heads=3, dim=10, rot=6, vdim=7, kv_rank=13, q_rank=11, ff=30), lat(3, heads=5, dim=9, rot=2, vdim=5, kv_rank=33, q_rank=3, yarn=(1.5, 20.0, 4.0, 1.0), ff=17),
                    lat(1, heads=1, dim=35, rot=34, vdim=21, kv_rank=50, q_rank=37, yarn=YARN)], vocab=77, width=50),
    "ones": lconfig([lat(3, heads=1, dim=1, rot=2, vdim=1, kv_rank=1, q_rank=1, scale=1.0, ff=1), lat(2, heads=1, dim=1, rot=2, vdim=1, kv_rank=1, q_rank=1, scale=1.0)], vocab=5, width=8),
    "scaling_by_one": lconfig([lat(1, yarn=(1.0, 64.0, 8.0, 1.0)), lat(3, yarn=(1.0, 4096.0, 32.0, 1.0))]),
    "ramp_of_no_width": lconfig([lat(1, rot=16, yarn=(4.0, 64.0, 1.0, 1.0)), lat(1, rot=16, base=10.0, yarn=(4.0, 2.0, 32.0, 16.0))]),
    "many_heads": lconfig([lat(3, heads=20, ff=16), lat(2, heads=33, dim=8, rot=4, vdim=8), lat(1, heads=16, yarn=YARN)], width=96),
    "large_heads": lconfig([lat(2, heads=2, dim=192, rot=64, vdim=256, kv_rank=96, q_rank=520), lat(1, heads=2, dim=32, rot=224, vdim=200, kv_rank=64, yarn=YARN, ff=520)], width=160),
    "large_latents": lconfig([lat(3, heads=4, dim=32, rot=64, vdim=32, kv_rank=704, q_rank=300, yarn=YARN), lat(2, heads=17, dim=16, rot=32, vdim=48, kv_rank=512, q_rank=64)], width=96),
    "real_proportions": lconfig([lat(1, heads=8, dim=128, rot=64, vdim=128, kv_rank=512, q_rank=768, yarn=YARN, ff=900)], vocab=1500, width=1040),
    "layers_without_feed_forward": lconfig([lat(2), lat(3), lat(2, kv_from=0), lat(1, ff=8)]),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(SIZES))
def test_sizes(name, dtype):
    cfg = SIZES[name]
    w = weights(cfg, 11)
    ids = tokens(83, cfg["vocab"], seed=2)
    fl = floats(w)
    want = so.forward(cfg, fl, ids)
    tol = bound(dtype, cfg, fl, ids, want)
    m = load(cfg, w, dtype)
    assert rel(whole(m, ids), want) < tol
    m.step([(1, ids[:60], 0, [])])
    assert rel(by_token(m, ids[60:], 1, 60), want[60:]) < tol
    assert rel(whole(m, ids[:20], stream=2), want[:20]) < tol       # (few tokens: the norms run inside the products or ahead of them)
    assert rel(whole(m, ids[20:22], stream=2, pos0=20), want[20:22]) < tol
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width", [50, 516, 1030, 1100, 2052, 4100, 8200])
def test_norms_of_every_width_and_row_count(width, dtype):
    """The norms (with and without a pending sublayer) run inside a product, a row per workgroup, several rows per workgroup or in
    pieces, by width and tokens: prompts of 300, 200 and 65, decode batches of 1 to 6."""
    cfg = lconfig([lat(1, ff=20), lat(3, q_rank=36), lat(2, q_rank=2 * (width // 4) + 1 if width < 2000 else 40)], width=width)
    w = weights(cfg, 13)
    fl = floats(w)
    m = load(cfg, w, dtype, max_streams=7, seq_len=320)
    ids = tokens(306, seed=7)
    want = so.forward(cfg, fl, ids)
    tol = bound(dtype, cfg, fl, ids, want)
    places = [0, 7, 8, 15, 63, 64, 190, 255, 256, 299]
    assert rel(whole(m, ids[:300], places), want[places]) < tol
    for n, st in ((200, 1), (65, 2), (64, 3), (17, 4), (3, 5)):
        assert rel(whole(m, ids[:n], None, st), want[:n]) < tol, n
    at = [300, 200, 65, 64, 17, 3]
    for n in (6, 5, 4, 3, 2, 1):
        out = m.step([(st, [ids[at[st]]], at[st], [0]) for st in range(n)])
        for st, o in enumerate(out):
            assert rel(o, want[at[st]]) < tol, (n, st)
            at[st] += 1
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("dim,rot,vdim", [(8, 4, 32), (24, 20, 64), (64, 24, 64), (90, 30, 128), (128, 64, 128), (40, 64, 80), (190, 60, 240)])
def test_long_prompts_at_every_head_size_of_the_prompt_attention(dim, rot, vdim, dtype):
    cfg = lconfig([lat(3, heads=3, dim=dim, rot=rot, vdim=vdim, yarn=YARN), lat(2, heads=2, dim=dim, rot=rot, vdim=vdim)])
    w = weights(cfg, 17)
    fl = floats(w)
    ids, other = tokens(430, seed=8), tokens(150, seed=9)
    want, want2 = so.forward(cfg, fl, ids), so.forward(cfg, fl, other)
    tol = bound(dtype, cfg, fl, ids, want)
    m = load(cfg, w, dtype, max_streams=2, seq_len=430)
    assert rel(whole(m, ids), want) < tol
    m.step([(0, ids[:100], 0, []), (1, other[:33], 0, [])])
    a, b = m.step([(0, ids[100:350], 100, list(range(250))), (1, other[33:], 33, list(range(117)))])
    assert rel(a, want[100:350]) < tol and rel(b, want2[33:]) < tol
    assert rel(by_token(m, ids[350:360], 0, 350), want[350:360]) < tol
    m.close()


# ---- cuts, batches, slots -------------------------------------------------------------------------------------------------------

@pytest.fixture(scope="module")
def base():
    cfg = lconfig(MIXED)
    w = weights(cfg, 21)
    ids = tokens(230, seed=9)
    m = load(cfg, w, "float32", max_streams=6, seq_len=400, max_step_tokens=128)
    yield cfg, w, ids, so.forward(cfg, floats(w), ids), m
    m.close()


@pytest.mark.parametrize("size", [2, 3, 15, 16, 17, 31, 63, 64, 65, 100, 127, 128, 129, 230])
def test_portions(base, size):
    _, _, ids, want, m = base
    got = np.concatenate([whole(m, ids[t:t + size], pos0=t) for t in range(0, len(ids), size)])
    assert rel(got, want) < F32_TOL


@pytest.mark.parametrize("first", [1, 2, 15, 16, 17, 31, 32, 33, 64, 65, 128, 200])
def test_prompt_then_decoding(base, first):
    _, _, ids, want, m = base
    whole(m, ids[:first], [])
    assert rel(by_token(m, ids[first:], pos0=first), want[first:]) < F32_TOL


def test_portions_between_decoded_tokens(base):
    _, _, ids, want, m = base
    at, rows = 0, []
    for n in (1, 1, 2, 1, 40, 1, 1, 1, 19, 2, 64, 1, 97):
        rows.append(whole(m, ids[at:at + n], pos0=at) if n > 1 else by_token(m, ids[at:at + 1], pos0=at))
        at += n
    assert rel(np.concatenate(rows), want[:at]) < F32_TOL


def test_unequal_requests_in_one_batch(base):
    cfg, w, _, _, m = base
    lens = [1, 2, 17, 64, 130, 5]
    seqs = [tokens(n + 12, seed=30 + n) for n in lens]
    wants = [so.forward(cfg, floats(w), s) for s in seqs]
    out = m.step([(i, s[:n], 0, list(range(n))) for i, (s, n) in enumerate(zip(seqs, lens))])
    for o, n, wt in zip(out, lens, wants):
        assert rel(o, wt[:n]) < F32_TOL
    alone = load(cfg, w, "float32", max_streams=1, seq_len=400)
    for i, (s, n) in enumerate(zip(seqs, lens)):
        assert rel(whole(alone, s[:n]), out[i]) < F32_TOL
    alone.close()
    for k in range(12):                                    # decoded together; one request drops out after every second step
        live = [i for i in range(6) if i >= k // 2]
        out = m.step([(i, [seqs[i][lens[i] + k]], lens[i] + k, [0]) for i in live])
        for o, i in zip(out, live):
            assert rel(o, wants[i][lens[i] + k]) < F32_TOL, (k, i)


def test_portions_whose_expanded_keys_do_not_fit_together(base):
    """Six streams with hundreds of earlier positions each go on by a few tokens: their keys are expanded group by group."""
    cfg, w, _, _, m = base
    lens = [390, 300, 10, 333, 256, 129]
    seqs = [tokens(n, seed=50 + n) for n in lens]
    wants = [so.forward(cfg, floats(w), s) for s in seqs]
    for cut in (3, 9):
        m.step([(i, s[:-cut], 0, []) for i, s in enumerate(seqs)])
        out = m.step([(i, s[-cut:], len(s) - cut, list(range(cut))) for i, s in enumerate(seqs)])
        for i, o in enumerate(out):
            assert rel(o, wants[i][-cut:]) < F32_TOL, (cut, i)


def test_prompts_beside_decoded_tokens(base):
    """One-token entries take the decode launches, the others the prompt launches: rows, ids and order are the caller's."""
    cfg, w, ids, want, m = base
    other, third = tokens(90, seed=77), tokens(12, seed=78)
    w2, w3 = so.forward(cfg, floats(w), other), so.forward(cfg, floats(w), third)
    whole(m, ids[:50], [], stream=2)
    whole(m, third[:11], [], stream=5)
    a, b, c, d = m.step([(2, [ids[50]], 50, [0]), (3, other, 0, list(range(90))), (0, ids[:1], 0, []), (5, third[11:], 11, [0])])
    assert rel(a, want[50]) < F32_TOL and rel(b, w2) < F32_TOL and c.shape == (0, 96) and rel(d, w3[11]) < F32_TOL
    assert rel(by_token(m, ids[1:4], 0, 1), want[1:4]) < F32_TOL


def test_streams_are_reused_without_traces_of_the_last_request(base):
    cfg, w, ids, want, m = base
    for n in (200, 9, 64, 1):
        m.reset(4)
        other = tokens(n, seed=n)
        whole(m, other, [], stream=4)
        by_token(m, other[:3], 4, n)
        m.reset(4)
        assert rel(whole(m, ids[:40], stream=4), want[:40]) < F32_TOL
        m.reset(4)
        assert rel(by_token(m, ids[:12], 4), want[:12]) < F32_TOL


def test_more_wanted_rows_than_one_logits_buffer():
    cfg = lconfig(MIXED[:2])
    w = weights(cfg, 22)
    ids = tokens(600, seed=4)
    m = load(cfg, w, "float32", max_streams=1, seq_len=600)
    assert rel(whole(m, ids), so.forward(cfg, floats(w), ids)) < F32_TOL
    m.close()


# ---- far keys -------------------------------------------------------------------------------------------------------------------
# Token KEY's key answers token QRY's query and nothing else does: one score stands out, and KEY's value is unlike any other.

KEY, QRY, PEAK = 1, 2, 14.0


def standout(kind, rotated, heads=5, dim=32, rot=8, kv_rank=40, q_rank=24, width=64, vocab=96):
    """rotated: the score goes through the last rotary pair, whose angle hardly changes over the distances of the tests."""
    span = (2 if rotated else dim) * (q_rank ** 0.5)
    cfg = lconfig([lat(kind, heads, dim, rot, 16, kv_rank, q_rank, base=1e9, scale=PEAK / (span * (4.0 if rotated else kv_rank ** 0.5)))], vocab, width)
    w = floats(weights(cfg, 8))
    rng = np.random.default_rng(4)
    w["embed"][:, :2] = 0.0
    w["embed"][KEY], w["embed"][QRY] = 0.0, 0.0
    w["embed"][KEY, 0] = w["embed"][QRY, 1] = 3.0
    for n in ("norm1", "mix.dq.norm", "mix.dkv.norm"):
        w["l0." + n][:] = 1.0
    pair = [rot - 2, rot - 1] if kind == 2 else [rot // 2 - 1, rot - 1]
    u = rng.choice([-1.0, 1.0], size=(heads, dim))
    dq, dkv, uq = w["l0.mix.dq"], w["l0.mix.dkv"], w["l0.mix.uq"].reshape(heads, dim + rot, q_rank)
    dq[:, 1], dkv[:, 0], dkv[0] = 0.0, 0.0, 0.0
    dq[0, 1] = dkv[0, 0] = 1.0
    uq *= 0.1
    uq[:, :, 0] = 0.0
    w["l0.mix.uk"] *= 0.1
    if rotated:
        dkv[kv_rank:] *= 0.1
        dkv[[kv_rank + p for p in pair], 0] = 4.0 / width ** 0.5      # (h is sqrt(width) in the mark's place)
        uq[:, [dim + p for p in pair], 0] = 1.0
        w["l0.mix.uk"][:, 0] = 0.0
    else:
        uq[:, :dim, 0] = u
        w["l0.mix.uk"][:, 0] = u.reshape(-1)
    w["l0.mix.uq"] = uq.reshape(heads * (dim + rot), q_rank)
    w["l0.mix.uv"][:, 0] = 2.0 * rng.standard_normal(heads * 16)
    return cfg, bits(w)


def _last_row(cfg, w, ids):
    """The oracle's logits of the last position of a one-layer model without feed-forward."""
    m, p, eps, kind = cfg["layers"][0]["mixer"], "l0.mix.", cfg["norm"]["eps"], cfg["layers"][0]["type"]
    adjacent, sink, gate = so.LATENT_KINDS[kind]
    H, d = m["heads"], m["dim"]
    h = so.norm_plain(w["embed"][ids], w["l0.norm1"], eps)
    c, r = so.latent_keys(h, m, w, p, eps, adjacent)
    q = (so.norm_plain(h[-1:] @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).reshape(H, d + m["rot_dim"])
    qr = so.rotate(np.broadcast_to(q[:, d:], (len(ids),) + q[:, d:].shape), m["rot"], adjacent)[-1]
    out = []
    for a in range(H):
        s = ((c @ w[p + "uk"].reshape(H, d, -1)[a].T) @ q[a, :d] + r @ qr[a]) * m["scale"]
        out.append(so.sink_softmax(s, w[p + "sink"][a] if sink else None) @ (c @ w[p + "uv"].reshape(H, m["vdim"], -1)[a].T))
    out = np.array(out)
    if gate:
        out *= so.sigmoid(h[-1] @ w[p + "g"].T)[:, None]
    x = w["embed"][ids[-1]] + so.norm_plain(out.reshape(-1) @ w[p + "o"].T, w["l0.norm1b"], eps)
    return so.norm_plain(x, w["final.norm"], eps) @ w["head"].T


@pytest.mark.parametrize("kind", [1, 2, 3])
def test_last_row_is_the_oracle(kind):
    for rotated in (False, True):
        cfg, w = standout(kind, rotated)
        ids, fl = tokens(40, seed=3), floats(w)
        assert np.allclose(_last_row(cfg, fl, ids), so.forward(cfg, fl, ids)[-1])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("rotated", [False, True])
@pytest.mark.parametrize("kind", [1, 2, 3])
def test_far_keys(kind, rotated, dtype):
    """Every key far back by itself, at the borders of key tiles, of prompt blocks and of a decode step's key splits."""
    cfg, w = standout(kind, rotated)
    fl = floats(w)
    m = load(cfg, w, dtype, max_streams=2, seq_len=1600, max_step_tokens=512)
    rng = np.random.default_rng(1)
    for n, places in ((1400, (0, 1, 15, 16, 31, 32, 33, 63, 64, 127, 128, 255, 256, 511, 512, 513, 703, 704, 1023, 1024, 1366, 1398)), (33, (0, 15, 16, 31)), (34, (0, 31, 32)), (2, (0,))):
        for at in places:
            ids = [3 + int(t) for t in rng.integers(0, 93, n)]
            ids[at], ids[-1] = KEY, QRY
            last = _last_row(cfg, fl, ids)
            gone = list(ids)
            gone[at] = 3
            assert rel(_last_row(cfg, fl, gone), last) > 2 * BF16_TOL        # the key shows
            assert rel(whole(m, ids, [n - 1], 0), last) < TOL[dtype], ("prompt", n, at)
            whole(m, ids[:-1], [], 1)
            assert rel(by_token(m, ids[-1:], 1, n - 1), last) < TOL[dtype], ("decoded", n, at)
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sink", [-20.0, 10.0, 12.0, 14.0, 60.0])
def test_sinks_below_beside_and_above_the_scores(sink, dtype):
    """A sink far above every score leaves almost nothing of the values; one far below changes nothing."""
    cfg, w = standout(3, False)
    w = floats(w)
    w["l0.mix.sink"][:] = sink + 0.5 * np.arange(5)
    w["l0.norm1b"] *= 20.0
    cfg["norm"]["eps"] = 1e-2                                # (the norm behind the mixer must not undo the sink's scaling)
    w = bits(w)
    fl = floats(w)
    m = load(cfg, w, dtype, max_streams=2, seq_len=600)
    for n in (3, 40, 500):
        ids = [3 + t % 90 for t in tokens(n, 93, seed=n)]
        ids[n // 2], ids[-1] = KEY, QRY
        want = _last_row(cfg, fl, ids)
        assert rel(whole(m, ids, [n - 1], 0), want) < TOL[dtype], n
        whole(m, ids[:-1], [], 1)
        assert rel(by_token(m, ids[-1:], 1, n - 1), want) < TOL[dtype], n
    m.close()


def test_a_sharing_layer_follows_its_owners_stream():
    """Layers that attend an earlier layer's latents: interleaved streams, freed and used again."""
    cfg = lconfig([lat(2, rot=16), lat(3), lat(2, rot=16, heads=4, kv_from=0), lat(2, rot=16), lat(2, rot=16, kv_from=3), lat(2, rot=16, kv_from=0, ff=16)])
    w = weights(cfg, 61)
    fl = floats(w)
    m = load(cfg, w, "float32", max_streams=3, seq_len=200)
    seqs = [tokens(n, seed=n) for n in (150, 40, 77)]
    wants = [so.forward(cfg, fl, s) for s in seqs]
    for rep in range(2):
        order = [0, 1, 2] if rep == 0 else [2, 0, 1]
        m.step([(st, seqs[i][:-20], 0, []) for st, i in enumerate(order)])
        for k in range(20):
            out = m.step([(st, [seqs[i][len(seqs[i]) - 20 + k]], len(seqs[i]) - 20 + k, [0]) for st, i in enumerate(order)])
            for o, i in zip(out, order):
                assert rel(o, wants[i][len(seqs[i]) - 20 + k]) < F32_TOL
    m.close()


# ---- latent attention as one mechanism among the others -------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_latent_layers_beside_other_mixers(dtype):
    """Another design's stack: gains of 1 + w, no norms behind the sublayers, tied output, gelu without biases, partly rotated keys, a sink
    without a gate, linear and windowed attention in the layers around."""
    from nanollama_amd.stack import LatentAttention, StackLayer, StackSpec, Yarn, load_stack_model
    from nanollama_amd.designs import DESIGNS
    from nanollama_amd.synth_stack import ganidra_config
    cfg = ganidra_config(96, 64, [gla(), par(ff=24), gla(ff=32)], embed_scale=1.5)
    w = weights(cfg, 5)
    spec = DESIGNS["Ganidra"](cfg, lambda n: w[n].shape)
    H, d, rot, v, kv, q, turn = 3, 16, 10, 12, 24, 20, 6
    t = LatentAttention(H, d, rot, v, q, kv, 0.2, 60.0, turn, False, Yarn(3.0, 50.0, 8.0, 1.0), None, True, False)
    spec.layers.insert(1, StackLayer(latent=t, ff=40))
    moved = {}
    for k, name in spec.tensors.items():
        p = k.split(".")
        if p[0] == "layers" and int(p[1]) >= 1:
            p[1] = str(int(p[1]) + 1)
        moved[".".join(p)] = name
    rng = np.random.default_rng(6)
    extra = {"norm1": 0.2 * rng.normal(size=64), "norm2": 0.2 * rng.normal(size=64), "latent.dq": rng.normal(size=(q, 64)) / 8, "latent.q_norm": 1 + 0.2 * rng.normal(size=q),
             "latent.uq": rng.normal(size=(H * (d + rot), q)) / q ** 0.5, "latent.dkv": rng.normal(size=(kv + rot, 64)) / 8, "latent.kv_norm": 1 + 0.2 * rng.normal(size=kv),
             "latent.uk": rng.normal(size=(H * d, kv)) / kv ** 0.5, "latent.uv": rng.normal(size=(H * v, kv)) / kv ** 0.5, "latent.o": rng.normal(size=(64, H * v)) / 6,
             "latent.sink": rng.uniform(0, 2, H), "ff.gate": rng.normal(size=(40, 64)) / 8, "ff.up": rng.normal(size=(40, 64)) / 8, "ff.down": rng.normal(size=(64, 40)) / 6}
    extra = bits(extra)
    moved.update({"layers.1." + k: "x." + k for k in extra})
    spec.tensors = moved
    full = dict(w, **{"x." + k: x for k, x in extra.items()})
    m = load_stack_model(spec, lambda n: ("BF16", full[n]), 0, 4, 256, dtype)
    fl, e, eps = floats(w), floats(extra), cfg["norm"]["eps"]
    rot_cfg = {"dims": turn, "base": 60.0, "scaling": {"factor": 3.0, "original": 50.0, "fast": 8.0, "slow": 1.0}}

    def forward(ids):
        x = fl["embed"][ids] * 1.5
        for i, L in enumerate(cfg["layers"]):
            p = f"l{i}."
            x = x + so.MIXERS[L["type"]](so.norm_one_plus(x, fl[p + "norm1"], eps), L["mixer"], fl, p + "mix.", eps)
            if L["mlp"] is not None:
                x = x + so.gated_mlp(so.norm_one_plus(x, fl[p + "norm2"], eps), fl, p + "mlp.")
            if i == 0:
                h = so.norm_one_plus(x, e["norm1"], eps)
                qs = (so.norm_plain(h @ e["latent.dq"].T, e["latent.q_norm"], eps) @ e["latent.uq"].T).reshape(len(ids), H, d + rot)
                ck = h @ e["latent.dkv"].T
                c, r, qr = so.norm_plain(ck[:, :kv], e["latent.kv_norm"], eps), so.rotate(ck[:, kv:], rot_cfg, False), so.rotate(qs[..., d:], rot_cfg, False)
                k, val = (c @ e["latent.uk"].T).reshape(-1, H, d), (c @ e["latent.uv"].T).reshape(-1, H, v)
                o = np.zeros((len(ids), H, v))
                for a in range(H):
                    s = np.where(np.tril(np.ones((len(ids),) * 2, bool)), (qs[:, a, :d] @ k[:, a].T + qr[:, a] @ r.T) * 0.2, -np.inf)
                    o[:, a] = so.sink_softmax(s, e["latent.sink"][a]) @ val[:, a]
                x = x + o.reshape(len(ids), -1) @ e["latent.o"].T
                x = x + so.gated_mlp(so.norm_one_plus(x, e["norm2"], eps), e, "ff.")
        return so.norm_one_plus(x, fl["final.norm"], eps) @ fl["embed"].T
    ids, other = tokens(90, seed=3), tokens(30, seed=4)
    want, want2 = forward(ids), forward(other)
    assert rel(whole(m, ids), want) < TOL[dtype]
    whole(m, ids[:50], [], 1)
    a, b = m.step([(2, other, 0, list(range(30))), (1, [ids[50]], 50, [0])])
    assert rel(a, want2) < TOL[dtype] and rel(b, want[50]) < TOL[dtype]
    assert rel(by_token(m, ids[51:], 1, 51), want[51:]) < TOL[dtype]
    m.close()


# ---- long decoding, generation --------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(dtype):
    cfg = lconfig(MIXED)
    w = weights(cfg, 41)
    ids = tokens(420, seed=13)
    fl = floats(w)
    want = so.forward(cfg, fl, ids)
    m = load(cfg, w, dtype, max_streams=2, seq_len=420, max_step_tokens=64)
    tol = bound(dtype, cfg, fl, ids, want)
    whole(m, ids[:7], [])
    assert rel(by_token(m, ids[7:], 0, 7), want[7:]) < tol
    got = np.concatenate([whole(m, ids[t:t + 50], stream=1, pos0=t) for t in range(0, 420, 50)])
    assert rel(got, want) < tol
    m.close()


@pytest.fixture(scope="module")
def gen():
    cfg = lconfig(MIXED)
    w = weights(cfg, 51)
    m = load(cfg, w, "float32", max_streams=3, seq_len=256)
    yield cfg, w, m
    m.close()


def test_greedy_generation_through_the_engine(gen):
    from nanollama_amd.engine import Engine, GenParams
    cfg, w, m = gen
    for n, k in ((1, 20), (5, 40), (33, 70)):
        prompt = tokens(n, seed=n)
        ids = Engine(m, eos_id=-1, rep_penalty=1.0).generate_ids(prompt, GenParams(max_tokens=k, temperature=0.0))
        assert ids == so.greedy(cfg, floats(w), prompt, k)


def test_generation_stops_at_the_sequence_limit(gen):
    from nanollama_amd.engine import Engine, GenParams
    ids = Engine(gen[2], eos_id=-1, rep_penalty=1.0).generate_ids(tokens(250), GenParams(max_tokens=50, temperature=0.0))
    assert len(ids) == 6                                   # positions 250 .. 255


def test_sampled_generation_matches_the_host_loop(gen):
    from nanollama_amd.engine import Engine, GenParams
    m = gen[2]
    for p in (GenParams(max_tokens=40, temperature=0.9, top_p=0.9), GenParams(max_tokens=40, temperature=0.7, top_p=1.0, top_k=12)):
        runs = [Engine(m, eos_id=-1, rep_penalty=1.2, seed=5, device_sampling=d).generate_ids(tokens(9, seed=3), p) for d in (True, False)]
        assert runs[0] == runs[1]


def test_scheduler_generates_like_single_requests(gen):
    from nanollama_amd.scheduler import Scheduler
    cfg, w, m = gen
    prompts = [tokens(n, seed=60 + n) for n in (3, 40, 1, 17, 8)]       # more requests than streams
    out = Scheduler(m).generate(prompts, 12)
    for p, o in zip(prompts, out):
        assert o == so.greedy(cfg, floats(w), p, 12)


def test_batched_argmax(gen):
    cfg, w, m = gen
    seqs = [tokens(n, seed=n) for n in (4, 9, 20)]
    for i, s in enumerate(seqs):
        whole(m, s[:-1], [], i)
    ids, lg = m.forward_batch([0, 1, 2], [s[-1] for s in seqs], [len(s) - 1 for s in seqs], want_logits=True)
    for i, s in enumerate(seqs):
        want = so.forward(cfg, floats(w), s)[-1]
        assert rel(lg[i], want) < F32_TOL and ids[i] == int(np.argmax(want))


def test_graph_replay_equals_eager_launches(gen):
    from nanollama_amd._lib import NL_FLAG_NO_GRAPH
    cfg, w, m = gen
    e = load(cfg, w, "float32", max_streams=3, seq_len=256, flags=NL_FLAG_NO_GRAPH)
    ids = tokens(60, seed=2)
    for rep in range(3):
        m.reset(0)
        e.reset(0)
        whole(m, ids[:20], [])
        whole(e, ids[:20], [])
        assert np.array_equal(by_token(m, ids[20:], 0, 20), by_token(e, ids[20:], 0, 20))
        a, b = (x.decode_greedy(3, 60, 50) for x in (m, e))
        assert a == b
    e.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n", [5, 17, 40, 64, 70])
def test_many_streams_in_one_decode_batch(n, dtype):
    cfg = lconfig([lat(2, rot=16), lat(3, heads=18, ff=24), lat(2, rot=16, kv_from=0)])
    w = weights(cfg, 71)
    seqs = [tokens(6 + i % 5 + (60 if i % 7 == 0 else 0), seed=i) for i in range(n)]
    m = load(cfg, w, dtype, max_streams=n, seq_len=80)
    fl = floats(w)
    m.step([(i, s[:-3], 0, []) for i, s in enumerate(seqs)])
    for k in (3, 2, 1):
        out = m.step([(i, [s[-k]], len(s) - k, [0] if i % 2 else []) for i, s in enumerate(seqs)])
    for i, s in enumerate(seqs):
        if i % 2:
            assert rel(out[i], so.forward(cfg, fl, s)[-1]) < TOL[dtype], i
    m.close()


# ---- the programs ---------------------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_runner(tmp_path, dtype):
    from nanollama_amd.synth_stack import write_folder
    cfg = lconfig(MIXED[:3])
    w = weights(cfg, 81)
    folder = write_folder(str(tmp_path / "m"), cfg, w)
    a, b = tokens(40, seed=1), tokens(9, seed=2)
    lines = [{"step": 0, "entries": [{"id": "a", "tokens": a[:38], "want": [0, 37]}, {"id": "b", "tokens": b[:7], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[38:39], "want": []}, {"id": "b", "tokens": b[7:8], "want": []}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[39:], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "c", "tokens": b, "want": [8]}], "end": ["c"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "64"],
                       input="".join(json.dumps(x) + "\n" for x in lines), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    fl = floats(w)
    wa, wb = so.forward(cfg, fl, a), so.forward(cfg, fl, b)
    tol = bound(dtype, cfg, fl, a, wa)
    read = lambda n: np.fromfile(str(tmp_path / f"{n}.f32"), "<f4").reshape(-1, 96)
    assert rel(read(0), wa[[0, 37]]) < tol and rel(read(2), wa[39]) < tol and rel(read(3), wb[8]) < tol
    assert not os.path.exists(str(tmp_path / "1.f32"))


def test_command_line_generates_from_a_folder(tmp_path):
    from nanollama_amd.synth_stack import write_folder
    cfg = lconfig(MIXED)
    w = weights(cfg, 91)
    folder = write_folder(str(tmp_path / "m"), cfg, w)
    prompt = tokens(6, seed=4)
    r = subprocess.run([sys.executable, "-m", "nanollama_amd", "--model", folder, "--dtype", "float32", "--prompt", " ".join(map(str, prompt)),
                        "--max-tokens", "10", "--temp", "0", "--rep-penalty", "1.0"], cwd=ROOT, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    ids = " ".join(map(str, so.greedy(cfg, floats(w), prompt, 10)))
    assert ids in r.stdout, (ids, r.stdout)
