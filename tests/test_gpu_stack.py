"""Layer-stack models (Ganidra) on the GPU against the float64 oracle (oracle/stack_oracle.py)."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from oracle import stack_oracle as so
from stack_models import BF16_TOL, F32_TOL, bits, config, floats, gla, load, par, rel, tokens, weights

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

TWO = [gla(), par(ff=48), gla(heads=3, dim=24, vdim=8, ff=40)]
TOL = {"float32": F32_TOL, "bfloat16": BF16_TOL}


def whole(m, ids, want=None, stream=0, pos0=0):
    return m.step([(stream, ids, pos0, list(range(len(ids))) if want is None else want)])[0]


def by_token(m, ids, stream=0, pos0=0):
    rows = []
    for i, t in enumerate(ids):
        m.forward(t, pos0 + i, stream)
        rows.append(m.state.logits.copy())
    return np.array(rows)


# ---- every mechanism by itself: one-layer models, the residual stream and the logits -------------------------------------------

def _zero(w, *names):
    for n in names:
        w[n] = np.zeros_like(w[n])


ALONE = {
    "embedding_and_head": (config([gla()]), lambda w: _zero(w, "l0.mix.o")),
    "gated_linear_attention": (config([gla(heads=3, dim=20, vdim=12, tau=5.0)]), None),
    "window_attention": (config([par(window=7, ls=1.0, rs=0.0)]), None),
    "attention_without_window": (config([par(window=0, ls=1.0, rs=0.0)]), None),
    "grouped_queries": (config([par(heads=6, kv=2, window=9, ls=1.0, rs=0.0)]), None),
    "linear_side_of_parallel": (config([par(ls=0.0, rs=1.0)]), None),
    "both_sides": (config([par(ls=-0.4, rs=2.0)]), None),
    "feed_forward": (config([gla(ff=72)]), lambda w: _zero(w, "l0.mix.o")),
    "loop": (config([gla(), gla(ff=32), gla()], loop=(1, 2, 3)), None),
    "eps_that_matters": (config([par(ff=32)], eps=0.3, embed_scale=0.2), None),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(ALONE))
def test_mechanism_alone(name, dtype):
    cfg, edit = ALONE[name]
    w = weights(cfg, 3)
    if edit:
        edit(w)
    ids = tokens(50, seed=5)
    want, layers = so.forward(cfg, floats(w), ids, want_layers=True)
    m = load(cfg, w, dtype)
    m.trace_layers(True)
    got = whole(m, ids)
    seen = m.layer_trace(len(ids))
    m.trace_layers(False)
    assert seen.shape == layers.shape
    for r in range(len(layers)):
        assert rel(seen[r], layers[r]) < TOL[dtype], r
    assert rel(got, want) < TOL[dtype]
    assert rel(by_token(m, ids, stream=1), want) < TOL[dtype]
    m.close()


def test_mechanism_tests_notice_a_wrong_oracle():
    """The one-layer models have the power to show a fault: the oracle with one constant off is far outside the tolerance."""
    ids = tokens(50, seed=5)
    for name, path, value in [("window_attention", ("left", "mask", "size"), 8), ("window_attention", ("left", "scale"), 0.2),
                              ("gated_linear_attention", ("tau",), 5.5), ("both_sides", ("right_scale",), 2.1)]:
        cfg, _ = ALONE[name]
        w = floats(weights(cfg, 3))
        off = copy.deepcopy(cfg)
        d = off["layers"][0]["mixer"]
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        assert rel(so.forward(off, w, ids), so.forward(cfg, w, ids)) > 100 * F32_TOL, name


# ---- sizes ----------------------------------------------------------------------------------------------------------------------

SIZES = {
    "odd": (config([gla(heads=3, dim=10, vdim=7), par(heads=3, kv=3, dim=18, vdim=22, window=5, rheads=1, rdim=9, rvdim=5, ff=30)], vocab=77, width=50), 3),
    "ones": (config([gla(heads=1, dim=1, vdim=1, tau=1.0), par(heads=1, kv=1, dim=2, vdim=1, window=1, scale=1.0, rheads=1, rdim=1, rvdim=2, tau=1.0, ls=1.0, rs=1.0, ff=1)],
                    vocab=5, width=8, loop=(0, 2, 1), embed_scale=1.0), 1),
    "values_wider_than_keys": (config([gla(heads=2, dim=16, vdim=80), par(heads=4, kv=2, dim=16, vdim=48, rdim=16, rvdim=128, ff=24)], width=96), 8),
    "keys_wider_than_values": (config([gla(heads=2, dim=112, vdim=16), par(heads=2, kv=2, dim=144, vdim=16, window=33, rdim=160, rvdim=16)], width=80), 16),
    "large_heads": (config([gla(heads=1, dim=256, vdim=256), par(heads=2, kv=1, dim=256, vdim=256, window=70, rheads=1, rdim=200, rvdim=136, ff=520)], width=160), 33),
    "wide": (config([gla(heads=4, dim=64, vdim=64, ff=700), par(heads=8, kv=2, dim=64, vdim=64, window=40, ff=900)], width=1040, vocab=1500), 16),
    "many_runs": (config([gla(), par(ff=16), gla(ff=16), par(window=3)], loop=(0, 4, 5)), 4),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(SIZES))
def test_sizes(name, dtype):
    cfg, rank = SIZES[name]
    w = weights(cfg, 11, rank)
    ids = tokens(83, cfg["vocab"], seed=2)
    want = so.forward(cfg, floats(w), ids)
    # (a network of many runs, or of single channels, amplifies roundings: bounded against a perturbed oracle instead of a constant)
    bent = dict(floats(w))
    bent["embed"] = bent["embed"] * (1 + np.random.default_rng(0).uniform(-1, 1, bent["embed"].shape) * (2.0 ** -8 if dtype == "bfloat16" else 2.0 ** -23))
    tol = max(TOL[dtype], 8 * rel(so.forward(cfg, bent, ids), want))
    m = load(cfg, w, dtype)
    assert rel(whole(m, ids), want) < tol
    m.step([(1, ids[:60], 0, [])])
    assert rel(by_token(m, ids[60:], 1, 60), want[60:]) < tol
    m.close()


# ---- cuts, batches, slots -------------------------------------------------------------------------------------------------------

@pytest.fixture(scope="module")
def base():
    cfg = config(TWO, loop=(0, 2, 2))
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


@pytest.mark.parametrize("first", [1, 2, 16, 23, 24, 25, 64, 65, 128, 200])
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


def test_prompt_beside_decoded_tokens(base):
    cfg, w, ids, want, m = base
    other = tokens(90, seed=77)
    w2 = so.forward(cfg, floats(w), other)
    whole(m, ids[:50], [], stream=2)
    a, b = m.step([(2, [ids[50]], 50, [0]), (3, other, 0, list(range(90)))])
    assert rel(a, want[50]) < F32_TOL and rel(b, w2) < F32_TOL


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


def test_positions_are_checked(base):
    from nanollama_amd._lib import NlError
    _, _, ids, _, m = base
    m.reset(5)
    with pytest.raises(NlError, match="goes on at position 0"):
        m.forward(ids[0], 3, 5)
    m.forward(ids[0], 0, 5)
    with pytest.raises(NlError, match="goes on at position 1"):
        m.forward(ids[0], 2, 5)
    with pytest.raises(NlError, match="out of range"):
        m.forward(96, 1, 5)
    with pytest.raises(NlError, match="appears twice"):
        m.step([(5, [1], 1, [0]), (5, [1], 1, [0])])
    with pytest.raises(NlError, match="outside"):
        m.step([(5, tokens(401), 0, [])])
    m.forward(ids[1], 1, 5)                                # still usable


def test_order_and_repetition_of_wanted_places(base):
    _, _, ids, want, m = base
    a, b = m.step([(0, ids[:30], 0, [29, 3, 3]), (1, ids[:20], 0, [])])
    assert rel(a, want[[29, 3, 3]]) < F32_TOL and b.shape == (0, 96)


def test_more_wanted_rows_than_one_logits_buffer(base):
    cfg, w, _, _, _ = base
    ids = tokens(600, seed=4)
    m = load(cfg, w, "float32", max_streams=1, seq_len=600)
    assert rel(whole(m, ids), so.forward(cfg, floats(w), ids)) < F32_TOL
    m.close()


# ---- far keys and window edges --------------------------------------------------------------------------------------------------
# Token KEY's key answers token QRY's query and nothing else does: one score stands out by PEAK, and KEY's value is unlike any other.

KEY, QRY, PEAK = 1, 2, 30.0


def standout(window, heads=8, dim=32, width=64, vocab=96, **kw):
    """The distance bias of the last head is the weakest (2^-8): far keys stay in play there."""
    cfg = config([par(heads=heads, kv=heads, dim=dim, vdim=16, window=window, scale=1.0, ls=1.0, rs=0.0, **kw)], vocab, width)
    w = floats(weights(cfg, 8))
    rng = np.random.default_rng(4)
    w["embed"][:, :2] = 0.0
    w["embed"][KEY], w["embed"][QRY] = 0.0, 0.0
    w["embed"][KEY, 0] = w["embed"][QRY, 1] = 3.0
    w["l0.norm1"][:] = 0.0
    w["l0.mix.left.q.norm"][:] = w["l0.mix.left.k.norm"][:] = np.sqrt(PEAK / dim)
    q, k = w["l0.mix.left.q"], w["l0.mix.left.k"]
    q *= 0.1
    k *= 0.1
    u = rng.choice([-1.0, 1.0], size=(heads * dim,))
    q[:, 1], k[:, 0] = u, u
    w["l0.mix.left.v"][:, 0] = 4.0 * rng.standard_normal(heads * 16)
    w = bits(w)
    return cfg, w


EDGES = [1, 2, 15, 16, 31, 32, 33, 47, 63, 64, 65, 95, 127]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("window", [2, 16, 33, 64, 100, 128])
def test_key_just_inside_and_outside_the_window(window, dtype):
    cfg, w = standout(window)
    m = load(cfg, w, dtype, max_streams=2, seq_len=600, max_step_tokens=64 if window < 64 else 0)
    fl = floats(w)
    off = copy.deepcopy(cfg)
    for at in (0, 5, 31, 32, 63, 64, 77):
        for dist, wrong in ((window - 1, window - 1), (window, window + 1)):
            if dist == 0:
                continue
            n = at + dist + 1
            ids = [3 + t % 90 for t in tokens(n, 93, seed=at + dist)]
            ids[at], ids[-1] = KEY, QRY
            want = so.forward(cfg, fl, ids)[-1]
            off["layers"][0]["mixer"]["left"]["mask"]["size"] = wrong
            assert wrong == 0 or rel(so.forward(off, fl, ids)[-1], want) > 2 * BF16_TOL      # one position off would show
            assert rel(whole(m, ids, [n - 1], 0), want) < TOL[dtype], ("prompt", at, dist)
            if n > 1:
                whole(m, ids[:-1], [], 1)
                assert rel(by_token(m, ids[-1:], 1, n - 1), want) < TOL[dtype], ("decoded", at, dist)
    m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_far_keys_in_a_long_window(dtype):
    """Every key far back by itself, at the borders of the ring's blocks and of a decode step's key splits."""
    cfg, w = standout(1500)
    fl = floats(w)
    n = 1400
    m = load(cfg, w, dtype, max_streams=2, seq_len=1600, max_step_tokens=512)
    rng = np.random.default_rng(1)
    for at in (0, 1, 15, 16, 31, 32, 63, 64, 127, 128, 129, 255, 256, 511, 512, 513, 700, 1023, 1024, 1200, n - 34, n - 2):
        ids = [3 + int(t) for t in rng.integers(0, 93, n)]
        ids[at], ids[-1] = KEY, QRY
        h = so.norm_one_plus(fl["embed"][ids] * 1.5, fl["l0.norm1"], 1e-5)
        last = _last_row(cfg, fl, h, ids)
        ids2 = list(ids)
        ids2[at] = 3
        assert rel(_last_row(cfg, fl, so.norm_one_plus(fl["embed"][ids2] * 1.5, fl["l0.norm1"], 1e-5), ids2), last) > 2 * BF16_TOL   # the key shows
        assert rel(whole(m, ids, [n - 1], 0), last) < TOL[dtype], ("prompt", at)
        whole(m, ids[:-1], [], 1)
        assert rel(by_token(m, ids[-1:], 1, n - 1), last) < TOL[dtype], ("decoded", at)
    m.close()


def _last_row(cfg, w, h, ids):
    """The oracle's logits of the last position of a one-layer model without a linear branch (its scale is 0)."""
    m, p, eps = cfg["layers"][0]["mixer"]["left"], "l0.mix.left.", cfg["norm"]["eps"]
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    q = so.rms((h[-1:] @ w[p + "q"].T).reshape(1, H, dk), eps) * w[p + "q.norm"]
    k = so.rms((h @ w[p + "k"].T).reshape(-1, H, dk), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T).reshape(-1, H, dv)
    dist = len(ids) - 1 - np.arange(len(ids))
    out = []
    for a in range(H):
        s = k[:, a] @ q[0, a] * m["scale"] - 2.0 ** (-8.0 * (a + 1) / H) * dist
        e = np.exp(s - s.max())
        out.append(e @ v[:, a] / e.sum())
    x = w["embed"][ids[-1]] * cfg["embedding"]["scale"] + (np.concatenate(out) * so.sigmoid(h[-1] @ w[p + "g"].T)) @ w[p + "o"].T
    return so.norm_one_plus(x, w["final.norm"], eps) @ w["embed"].T


def test_last_row_is_the_oracle():
    cfg, w = standout(64)
    ids = tokens(40, 93, seed=3)
    fl = floats(w)
    h = so.norm_one_plus(fl["embed"][ids] * 1.5, fl["l0.norm1"], 1e-5)
    assert np.allclose(_last_row(cfg, fl, h, ids), so.forward(cfg, fl, ids)[-1])


# ---- recurrent state ------------------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("bias", [40.0, 3.0, -10.0, -300.0])
def test_decays_from_none_to_total(bias, dtype):
    """bias 40: the state keeps everything; -10: beyond the range in which a sub-chunk's decays factor; -300: it forgets at once."""
    cfg = config([gla(heads=2, dim=24, vdim=16, tau=1.0), par(rdim=24, tau=1.0, ls=0.0, rs=1.0)])
    w = floats(weights(cfg, 5))
    for n in ("l0.mix.a2.b", "l1.mix.right.a2.b"):
        w[n] = w[n] * 0.3 + bias
        w[n][::5] = 6.0                                    # beside slow channels, whose products must not suffer
    w = bits(w)
    ids = tokens(150, seed=6)
    want = so.forward(cfg, floats(w), ids)
    m = load(cfg, w, dtype)
    assert rel(whole(m, ids), want) < TOL[dtype]
    whole(m, ids[:70], [], 1)
    assert rel(by_token(m, ids[70:], 1, 70), want[70:]) < TOL[dtype]
    m.close()


def test_state_carries_the_first_token():
    """A state that barely decays: the first token's mark is there hundreds of tokens later, whatever lies between."""
    cfg = config([gla(heads=1, dim=16, vdim=16, tau=64.0)])
    w = floats(weights(cfg, 5))
    w["l0.mix.a2.b"][:] = 9.0
    w["l0.mix.a2"][:] = 0.0
    w["l0.mix.v"] *= 0.02
    w["embed"][:, 0] = 0.0
    w["embed"][KEY] = 0.0
    w["embed"][KEY, 0] = 3.0
    w["l0.mix.v"][:, 0] = 5.0 * np.random.default_rng(2).standard_normal(16)
    w = bits(w)
    fl = floats(w)
    ids = [KEY] + [3 + t % 90 for t in tokens(399, 93, seed=8)]
    want = so.forward(cfg, fl, ids)
    assert rel(so.forward(cfg, fl, [4] + ids[1:])[-1], want[-1]) > 100 * F32_TOL
    m = load(cfg, w, "float32", seq_len=400)
    assert rel(whole(m, ids), want) < F32_TOL
    for cut in (1, 15, 16, 17, 64, 100):
        whole(m, ids[:cut], [], 1)
        assert rel(whole(m, ids[cut:], stream=1, pos0=cut), want[cut:]) < F32_TOL, cut
    whole(m, ids[:2], [], 1)
    assert rel(by_token(m, ids[2:], 1, 2), want[2:]) < F32_TOL
    m.close()


def test_loop_passes_have_their_own_state_and_ring():
    cfg = config([par(window=11, ff=24), gla()], loop=(0, 2, 3))
    w = weights(cfg, 31)
    fl = floats(w)
    ids = tokens(70, seed=12)
    want = so.forward(cfg, fl, ids)
    flat = copy.deepcopy(cfg)
    flat["loop"]["times"] = 2
    assert rel(so.forward(flat, fl, ids), want) > 100 * F32_TOL
    m = load(cfg, w, "float32")
    assert rel(whole(m, ids), want) < F32_TOL
    assert rel(by_token(m, ids, 1), want) < F32_TOL
    s = [m.debug_read(f"state{r}", 10000, 1) for r in range(6)]
    for a in range(6):
        for b in range(a):
            assert s[a].shape != s[b].shape or not np.array_equal(s[a], s[b])
    m.close()


# ---- long decoding, generation --------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_around_the_ring(dtype):
    cfg = config([par(window=30, ff=24), gla()])
    w = weights(cfg, 41)
    ids = tokens(420, seed=13)
    want = so.forward(cfg, floats(w), ids)
    m = load(cfg, w, dtype, max_streams=2, seq_len=2000, max_step_tokens=64)     # ring of 128 positions
    whole(m, ids[:7], [])
    assert rel(by_token(m, ids[7:], 0, 7), want[7:]) < TOL[dtype]
    got = np.concatenate([whole(m, ids[t:t + 50], stream=1, pos0=t) for t in range(0, 420, 50)])
    assert rel(got, want) < TOL[dtype]
    m.close()


@pytest.fixture(scope="module")
def gen():
    cfg = config(TWO, loop=(1, 3, 2), embed_scale=1.0)
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
    _, _, m = gen
    ids = Engine(m, eos_id=-1, rep_penalty=1.0).generate_ids(tokens(250), GenParams(max_tokens=50, temperature=0.0))
    assert len(ids) == 6                                   # positions 250 .. 255


def test_sampled_generation_matches_the_host_loop(gen):
    from nanollama_amd.engine import Engine, GenParams
    _, _, m = gen
    for p in (GenParams(max_tokens=40, temperature=0.9, top_p=0.9), GenParams(max_tokens=40, temperature=0.7, top_p=1.0, top_k=12),
              GenParams(max_tokens=40, temperature=0.0)):
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


def test_many_streams_in_one_decode_batch():
    cfg = config([gla(), par(heads=2, kv=1, ff=24)])
    w = weights(cfg, 71)
    n = 70                                                 # more than one launch sequence holds
    seqs = [tokens(6 + i % 5, seed=i) for i in range(n)]
    m = load(cfg, w, "float32", max_streams=n, seq_len=32)
    fl = floats(w)
    m.step([(i, s[:-3], 0, []) for i, s in enumerate(seqs)])
    for k in (3, 2, 1):
        out = m.step([(i, [s[-k]], len(s) - k, [0] if i % 2 else []) for i, s in enumerate(seqs)])
    for i, s in enumerate(seqs):
        if i % 2:
            assert rel(out[i], so.forward(cfg, fl, s)[-1]) < F32_TOL, i
    m.close()


# ---- the programs ---------------------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_runner(tmp_path, dtype):
    from nanollama_amd.synth_stack import write_folder
    cfg = config(TWO, loop=(0, 2, 2))
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
    wa, wb = so.forward(cfg, floats(w), a), so.forward(cfg, floats(w), b)
    read = lambda n: np.fromfile(str(tmp_path / f"{n}.f32"), "<f4").reshape(-1, 96)
    assert rel(read(0), wa[[0, 37]]) < TOL[dtype] and rel(read(2), wa[39]) < TOL[dtype] and rel(read(3), wb[8]) < TOL[dtype]
    assert not os.path.exists(str(tmp_path / "1.f32"))


def test_command_line_generates_from_a_folder(tmp_path):
    from nanollama_amd.synth_stack import write_folder
    cfg = config(TWO, embed_scale=1.0)
    w = weights(cfg, 91)
    folder = write_folder(str(tmp_path / "m"), cfg, w)
    prompt = tokens(6, seed=4)
    r = subprocess.run([sys.executable, "-m", "nanollama_amd", "--model", folder, "--dtype", "float32", "--prompt", " ".join(map(str, prompt)),
                        "--max-tokens", "10", "--temp", "0", "--rep-penalty", "1.0"], cwd=ROOT, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    ids = " ".join(map(str, so.greedy(cfg, floats(w), prompt, 10)))
    assert ids in r.stdout, (ids, r.stdout)
