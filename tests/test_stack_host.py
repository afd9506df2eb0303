"""Host side of the layer-stack models without a GPU: the library's surface, the design's reader, weight files, the scheduler, the
trace runner, the command line -- and the oracle's own consistency."""
import copy
import ctypes
import json
import os
import re
import struct
from types import SimpleNamespace

import numpy as np
import pytest

from nanollama_amd import _lib, cli, registry, trace
from nanollama_amd.designs import DESIGNS
from nanollama_amd.safetensors import SafetensorsFile, from_bf16, save, to_bf16
from nanollama_amd.scheduler import Scheduler
from nanollama_amd.synth_stack import write_folder
from nanollama_amd.tokenizer import IdTokenizer
from oracle import stack_oracle as so
from stack_models import F32_TOL, config, floats, gla, lat, lconfig, par, rel, tokens, weights

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ---- library ------------------------------------------------------------------------------------------------------------------

def test_stack_library_exports_its_surface():
    _lib.build(family="stack")
    L = ctypes.CDLL(_lib.STACK_LIB_PATH)
    text = open(os.path.join(ROOT, "include", "nanollama_stack.h")).read()
    declared = re.findall(r"NL_API\s+[\w\s\*]+?\b(nl_\w+)\s*\(", text)
    listed = set(re.findall(r"\bnl_\w+\b", text[:text.index("#ifndef")])) - {"nl_create_stack"}
    shared = {n for n in listed if n in _lib.EXPORTS}
    missing = [n for n in list(declared) + sorted(shared) + _lib.STACK_EXPORTS if not hasattr(L, n)]
    assert not missing, missing
    assert len(declared) == 3 and len(shared) >= 18


def test_the_sources_of_each_library_are_hashed_as_the_makefile_does():
    L = ctypes.CDLL(_lib.STACK_LIB_PATH)
    L.nl_build_info.restype = ctypes.c_char_p
    assert L.nl_build_info().decode().startswith("src=" + _lib.source_sha(_lib.source_files("stack")) + " ")


def _create(cfg, w, **kw):
    spec = DESIGNS[cfg["architecture"]](cfg, lambda n: w[n].shape)
    from nanollama_amd.stack import load_stack_model
    return load_stack_model(spec, lambda n: ("BF16", w[n]), **kw)


def test_create_fails_loudly_without_a_gpu_and_on_bad_shapes():
    cfg = config([gla()])
    w = weights(cfg)
    if _lib.stack_lib().nl_device_count() == 0:
        with pytest.raises(_lib.NlError, match="no HIP device"):
            _create(cfg, w)
    for bad, text in ((config([par(heads=3, kv=2)]), "attention sizes"), (config([gla(dim=300)]), "up to 256"), (config([gla(tau=0.0)]), "linear attention"),
                      (config([gla()], loop=(0, 2, 2)), "loop range"), (config([par(window=-3)]), "attention sizes")):
        with pytest.raises(_lib.NlError, match=text):
            _create(bad, weights(bad))
    for layers, text in (([lat(dim=250)], "up to 256"), ([lat(vdim=300)], "up to 256"), ([lat(kv_rank=760)], "up to 768"), ([lat(base=0.0)], "latent attention sizes"),
                         ([lat(heads=0)], "no mixer"), ([lat(1, yarn=(-1.0, 9.0, 2.0, 1.0))], "rotary scaling"), ([lat(2), lat(2, kv_rank=40, kv_from=0)], "kv_from"),
                         ([lat(2), lat(2, kv_from=1)], "kv_from"), ([lat(2), lat(2, kv_from=0), lat(2, kv_from=1)], "kv_from")):
        bad = lconfig(layers)
        with pytest.raises(_lib.NlError, match=text):
            _create(bad, weights(bad))
    with pytest.raises(ValueError, match="dtype"):
        _create(cfg, w, dtype="float16")


# ---- design, registry, weight files --------------------------------------------------------------------------------------------

def test_design_reads_every_size_and_constant():
    cfg = config([gla(heads=3, dim=10, vdim=6, tau=5.0), par(heads=6, kv=2, dim=8, vdim=12, window=9, scale=0.31, rheads=4, rdim=2, rvdim=3, tau=2.5, ls=0.2, rs=0.9, ff=22)],
                 vocab=41, width=26, loop=(0, 1, 4), eps=2e-4, embed_scale=3.25)
    w = weights(cfg, rank=7)
    s = DESIGNS["Ganidra"](cfg, lambda n: w[n].shape)
    assert (s.vocab, s.dim, s.eps, s.embed_scale, s.loop, s.runs()) == (41, 26, 2e-4, 3.25, (0, 1, 4), [0, 0, 0, 0, 1])
    a, b = s.layers
    assert a.attn is None and (a.lin.heads, a.lin.dim, a.lin.vdim, a.lin.rank, a.lin.tau, a.lin.mix_scale, a.ff) == (3, 10, 6, 7, 5.0, 1.0, 0)
    assert (b.attn.heads, b.attn.kv_heads, b.attn.dim, b.attn.vdim, b.attn.window, b.attn.scale, b.attn.mix_scale) == (6, 2, 8, 12, 9, 0.31, 0.2)
    assert b.attn.qk_norm and b.attn.gate and b.attn.distance_bias
    assert (b.lin.heads, b.lin.dim, b.lin.vdim, b.lin.tau, b.lin.mix_scale, b.ff) == (4, 2, 3, 2.5, 0.9, 22)
    assert sorted(s.tensors.values()) == sorted(w)         # every tensor of the file has exactly one place
    no_loop = copy.deepcopy(cfg)
    del no_loop["loop"]
    assert DESIGNS["Ganidra"](no_loop, lambda n: w[n].shape).runs() == [0, 1]
    no_mask = copy.deepcopy(cfg)
    no_mask["layers"][1]["mixer"]["left"]["mask"] = None
    assert DESIGNS["Ganidra"](no_mask, lambda n: w[n].shape).layers[1].attn.window == 0


def test_latent_design_reads_every_size_and_constant():
    cfg = lconfig([lat(2, heads=3, dim=10, rot=6, vdim=7, kv_rank=13, q_rank=11, base=321.0, scale=0.37, ff=30), lat(1, heads=5, dim=12, rot=4, yarn=(1.5, 20.0, 4.0, 0.5)),
                   lat(3, heads=2, kv_rank=9, yarn=(8.0, 640.0, 16.0, 2.0), ff=9), lat(2, heads=4, dim=8, rot=6, kv_rank=13, base=321.0, kv_from=0)], vocab=41, width=26, eps=3e-3)
    w = weights(cfg)
    s = DESIGNS["Pabalix"](cfg, lambda n: w[n].shape)
    assert (s.vocab, s.dim, s.eps, s.embed_scale, s.loop, s.plain_norm, s.post_norm, s.untied) == (41, 26, 3e-3, 1.0, None, True, True, True)
    a, b, c, d = (l.latent for l in s.layers)
    assert (a.heads, a.dim, a.rot_dim, a.vdim, a.q_rank, a.kv_rank, a.scale, a.rope_base, a.rot_dims) == (3, 10, 6, 7, 11, 13, 0.37, 321.0, 6)
    assert [(x.adjacent_pairs, x.sink, x.gate, x.kv_from) for x in (a, b, c, d)] == [(True, False, False, None), (False, False, False, None), (False, True, True, None), (True, False, False, 0)]
    assert a.yarn is None and (b.yarn.factor, b.yarn.original, b.yarn.fast, b.yarn.slow) == (1.5, 20.0, 4.0, 0.5) and c.yarn.original == 640.0
    assert [(l.ff, l.ff_bias) for l in s.layers] == [(30, True), (0, False), (9, True), (0, False)] and s.layers[0].ff_act == "silu"
    assert sorted(s.tensors.values()) == sorted(w)         # every tensor of the file has exactly one place
    for edit in (lambda x: x["layers"][0].update(type="latent_attention_9"), lambda x: x["layers"][0].update(mlp={"kind": "experts", "ff": 8})):
        bad = copy.deepcopy(cfg)
        edit(bad)
        with pytest.raises(ValueError, match="unknown"):
            DESIGNS["Pabalix"](bad, lambda n: w[n].shape)


def test_unknown_designs_and_layers_are_refused(tmp_path):
    cfg = config([gla()])
    w = weights(cfg)
    other = dict(cfg, architecture="Somethingelse")
    with pytest.raises(ValueError, match="Somethingelse.*Ganidra"):
        registry.read_spec(write_folder(str(tmp_path / "a"), other, w))
    for edit in (lambda c: c["layers"][0].update(type="mamba"), lambda c: c["layers"][0].update(mlp={"kind": "experts", "ff": 8})):
        bad = copy.deepcopy(cfg)
        edit(bad)
        with pytest.raises(ValueError, match="unknown"):
            registry.read_spec(write_folder(str(tmp_path / "b"), bad, w))
    assert "Ganidra" in registry.architectures() and not registry.is_model_folder(str(tmp_path))


def test_safetensors_round_trip_and_damaged_files(tmp_path):
    p = str(tmp_path / "x.safetensors")
    x = {"a": to_bf16(np.float32([[1.0, -2.5], [3.0, 0.1]])), "b": np.float32([1, 2, 3]), "c": np.int32([[7]])}
    save(p, x)
    f = SafetensorsFile(p)
    assert list(f.names()) == ["a", "b", "c"] and f.shape("a") == (2, 2) and "b" in f and "d" not in f
    for n, tag in (("a", "BF16"), ("b", "F32"), ("c", "I32")):
        t, y = f.get(n)
        assert t == tag and np.array_equal(y, x[n])
    raw = open(p, "rb").read()
    n = struct.unpack("<Q", raw[:8])[0]
    for bad in (raw[:6], struct.pack("<Q", 1 << 40) + raw[8:], raw[:-4], raw[:8] + raw[8:8 + n].replace(b"[0, 8]", b"[0, 9]") + raw[8 + n:]):
        open(p + "2", "wb").write(bad)
        with pytest.raises(ValueError):
            SafetensorsFile(p + "2")


def test_bfloat16_rounding_is_to_nearest_even():
    x = np.float32([1.0, 1.00390625, 1.01171875, -1.00390625, 3.0e38, 0.0])
    y = from_bf16(to_bf16(x))
    assert np.array_equal(y[:4], np.float32([1.0, 1.0, 1.015625, -1.0])) and np.all(np.abs(y - x) <= np.abs(x) * 2.0 ** -8)


# ---- scheduler, trace runner, command line -------------------------------------------------------------------------------------

class FakeModel:
    """Logits are a function of the stream's whole token history."""

    def __init__(self, vocab=50, streams=2, seq_len=40):
        self.config = SimpleNamespace(vocab_size=vocab, seq_len=seq_len)
        self.max_streams, self.hist, self.batches = streams, {}, []

    def reset(self, stream=0):
        self.hist[stream] = []

    def logits(self, hist):
        out = np.zeros(self.config.vocab_size, np.float32)
        out[(sum(hist) * 7 + len(hist)) % self.config.vocab_size] = 1.0
        return out

    def step(self, entries):
        self.batches.append(len(entries))
        out = []
        for stream, toks, pos0, want in entries:
            assert pos0 == len(self.hist[stream])
            rows = []
            for t in toks:
                self.hist[stream].append(t)
                rows.append(self.logits(self.hist[stream]))
            out.append(np.array([rows[k] for k in want], np.float32).reshape(len(want), self.config.vocab_size))
        return out

    def close(self):
        pass


def test_scheduler_assigns_and_frees_streams():
    m = FakeModel()
    s = Scheduler(m)
    a = s.step([("a", [1, 2, 3], [2, 0]), ("b", [4], [])])
    assert a[0].shape == (2, 50) and a[1].shape == (0, 50) and s.position("a") == 3 and sorted(s.live()) == ["a", "b"]
    with pytest.raises(RuntimeError, match="0 of 2 streams"):
        s.step([("c", [1], [])])
    with pytest.raises(ValueError, match="twice"):
        s.step([("a", [1], []), ("a", [1], [])])
    s.finish(["a"])
    c = s.step([("b", [5], [0]), ("c", [9, 9], [1])])
    assert np.array_equal(c[0][0], m.logits([4, 5])) and np.array_equal(c[1][0], m.logits([9, 9]))


def test_scheduler_generates_more_requests_than_streams():
    m = FakeModel(streams=3)
    prompts = [tokens(n, 50, seed=n) for n in (1, 5, 2, 9, 4, 3, 38)]
    out = Scheduler(m).generate(prompts, 6)
    for p, o in zip(prompts, out):
        h = list(p)
        for t in o:
            assert t == int(np.argmax(m.logits(h)))
            h.append(t)
        assert len(o) == min(6, 40 - len(p) + 1)
    assert max(m.batches) == 3


def test_step_without_a_ragged_step_cuts_behind_every_wanted_place():
    from nanollama_amd.model import HipModel
    m = HipModel(SimpleNamespace(vocab_size=4, seq_len=100), None, 2, None)
    calls = []

    def prefill(toks, pos0=0, stream=0, want_logits=True):
        calls.append((list(toks), pos0, stream, want_logits))
        m.state.logits[:] = len(calls)
    m.prefill = prefill
    out = m.step([(1, [5, 6, 7, 8], 10, [0, 2]), (0, [9], 0, [])])
    assert calls == [([5], 10, 1, True), ([6, 7], 11, 1, True), ([8], 13, 1, False), ([9], 0, 0, False)]
    assert out[0][:, 0].tolist() == [1, 2] and out[1].shape == (0, 4)


def test_trace_runner_protocol(tmp_path, monkeypatch, capsys):
    import io
    m = FakeModel(streams=8)
    seen = {}
    monkeypatch.setattr(registry, "load_model", lambda path, **kw: seen.update(kw, path=path) or m)
    lines = [{"step": 7, "entries": [{"id": "x", "tokens": [1, 2, 3], "want": [2, 0]}, {"id": "y", "tokens": [4], "want": [0]}], "end": ["y"]},
             {"step": 8, "entries": [{"id": "x", "tokens": [6], "want": []}], "end": []},
             {"step": 9, "entries": [], "end": ["x"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("".join(json.dumps(x) + "\n" for x in lines)))
    assert trace.main(["--model", "folder", "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "40"]) == 0
    assert capsys.readouterr().out.split("\n")[:3] == ["done 7", "done 8", "done 9"]
    got = np.fromfile(str(tmp_path / "7.f32"), "<f4").reshape(3, 50)
    assert np.array_equal(got, np.array([m.logits([1, 2, 3]), m.logits([1]), m.logits([4])]))
    assert os.listdir(str(tmp_path)) == ["7.f32"] and seen["dtype"] == "float32" and seen["seq_len"] == 40 and seen["path"] == "folder"
    assert os.access(os.path.join(ROOT, "bin", "trace_run"), os.X_OK)


def test_id_prompts():
    t = IdTokenizer(50)
    assert t.encode(" 1 2\n49 ") == [1, 2, 49] and t.decode_token_bytes(7) == b"7 " and t.decode([1, 2]) == "1 2 "
    for bad in ("hello", "50", "-1", ""):
        with pytest.raises(ValueError):
            t.encode(bad)


def test_command_line_on_a_folder(tmp_path, capsys):
    cfg = config([gla()])
    folder = write_folder(str(tmp_path / "m"), cfg, weights(cfg))
    assert cli.main(["--model", folder, "--list-tensors"]) == 0
    assert "l0.mix.a2.b" in capsys.readouterr().out
    if _lib.stack_lib().nl_device_count() == 0:
        assert cli.main(["--model", folder, "--prompt", "1 2"]) == 1
        assert "no HIP device" in capsys.readouterr().err
    os.remove(os.path.join(folder, "model.safetensors"))
    assert cli.main(["--model", folder, "--prompt", "1 2"]) == 1


# ---- the oracle against itself --------------------------------------------------------------------------------------------------

def test_oracle_recurrence_is_its_closed_form():
    """S_t = sum_s (prod_{r = s+1..t} alpha_r) k_s v_s^T, written out."""
    rng = np.random.default_rng(0)
    q, k, v, al = rng.normal(size=(9, 4)), rng.normal(size=(9, 4)), rng.normal(size=(9, 3)), rng.uniform(0.2, 1, (9, 4))
    o, S = so.gated_recurrence(q, k, v, al)
    for t in range(9):
        want = sum(np.outer(np.prod(al[s + 1:t + 1], axis=0) * k[s], v[s]) for s in range(t + 1))
        assert np.allclose(o[t], want.T @ q[t])
    o2, _ = so.gated_recurrence(q[5:], k[5:], v[5:], al[5:], so.gated_recurrence(q[:5], k[:5], v[:5], al[:5])[1])
    assert np.allclose(o2, o[5:])


def test_oracle_attention_sees_exactly_the_window():
    rng = np.random.default_rng(1)
    q, k = rng.normal(size=(12, 4)), rng.normal(size=(12, 4))
    a = so.attention_weights(q, k, 0.5, 0.25, 5)
    for i in range(12):
        assert np.allclose(a[i].sum(), 1) and np.array_equal(np.nonzero(a[i])[0], np.arange(max(0, i - 4), i + 1))
        j = np.arange(max(0, i - 4), i + 1)
        s = np.exp(0.5 * k[j] @ q[i] - 0.25 * (i - j))
        assert np.allclose(a[i, j], s / s.sum())
    assert np.all(np.tril(so.attention_weights(q, k, 0.5, 0.0, None)) > -1) and np.count_nonzero(so.attention_weights(q, k, 0.5, 0.0, None)) == 78


def test_oracle_is_causal_and_loops_differ_from_repeated_layers():
    cfg = config([gla(), par(ff=16)], loop=(0, 2, 2))
    w = floats(weights(cfg, 2))
    ids = tokens(20, seed=1)
    full = so.forward(cfg, w, ids)
    assert rel(so.forward(cfg, w, ids[:13]), full[:13]) < 1e-12
    assert so.layer_runs(cfg) == [(0, False), (1, False), (0, True), (1, False)]
    again = copy.deepcopy(cfg)
    again["layers"] = cfg["layers"] * 2
    del again["loop"]
    w2 = dict(w, **{k.replace("l0.", "l2.", 1).replace("l1.", "l3.", 1): v for k, v in w.items() if k[:2] in ("l0", "l1")})
    assert rel(so.forward(again, w2, ids), full) > 1e-3      # (the passes of a loop start from x + the embedding)


def test_oracle_rotation_depends_on_distance_alone():
    rng = np.random.default_rng(2)
    q, k = np.tile(rng.normal(size=10), (30, 1)), np.tile(rng.normal(size=10), (30, 1))
    yarn = {"factor": 4.0, "original": 20.0, "fast": 8.0, "slow": 1.0}
    for rot in ({"dims": 8, "base": 50.0}, {"dims": 8, "base": 50.0, "scaling": yarn}):
        for adjacent in (False, True):
            s = so.rotate(q, rot, adjacent) @ so.rotate(k, rot, adjacent).T
            for d in range(29):
                assert np.allclose(np.diagonal(s, -d), s[d, 0])
            far = (1.0 if "scaling" not in rot else 0.1 * np.log(4.0) + 1.0) ** 2
            assert np.allclose(s[0, 0], far * (q[0, :8] @ k[0, :8]) + q[0, 8:] @ k[0, 8:])


def test_oracle_yarn_leaves_fast_pairs_and_stretches_slow_ones():
    rot = {"dims": 64, "base": 10000.0}
    f, one = so.rotary_frequencies(rot)
    y, m = so.rotary_frequencies(dict(rot, scaling={"factor": 8.0, "original": 4096.0, "fast": 32.0, "slow": 1.0}))
    turns = f * 4096.0 / (2 * np.pi)
    assert one == 1.0 and np.isclose(m, 1.0 + 0.1 * np.log(8.0))
    ratio = y / f
    assert np.allclose(ratio[turns > 40], 1.0) and np.allclose(ratio[turns < 0.8], 1 / 8.0) and np.all(np.diff(ratio) <= 1e-12)
    assert np.any((ratio < 0.9) & (ratio > 0.2))


def test_oracle_sink_is_one_more_score_without_a_value():
    rng = np.random.default_rng(3)
    s = rng.normal(size=(4, 6))
    s[0, 3:] = -np.inf
    for sink in (-50.0, 0.3, 40.0):
        e = np.exp(np.concatenate([s, np.full((4, 1), sink)], axis=1))
        assert np.allclose(so.sink_softmax(s, sink), e[:, :6] / e.sum(axis=1, keepdims=True))
    assert np.allclose(so.sink_softmax(s).sum(axis=-1), 1.0)


def test_oracle_latent_model_is_causal_and_small_changes_of_a_constant_show():
    """The mixed latent model has the power to show a fault: the oracle with one thing off is far outside the float32 tolerance."""
    yarn = (4.0, 64.0, 8.0, 1.0)
    cfg = lconfig([lat(2, rot=16, ff=16), lat(1, rot=16, yarn=yarn), lat(3, rot=16, yarn=yarn), lat(2, rot=16, kv_from=0)])
    w, ids = floats(weights(cfg, 4)), tokens(60, seed=6)
    full = so.forward(cfg, w, ids)
    assert rel(so.forward(cfg, w, ids[:23]), full[:23]) < 1e-12

    def off(edit):
        c = copy.deepcopy(cfg)
        edit(c["layers"])
        return rel(so.forward(c, w, ids), full)
    mix = lambda i, **kw: (lambda L: L[i]["mixer"].update(kw))
    rot = lambda i, **kw: (lambda L: L[i]["mixer"]["rot"].update(kw))
    scl = lambda i, **kw: (lambda L: L[i]["mixer"]["rot"]["scaling"].update(kw))
    kind = lambda i, t: (lambda L: L[i].update(type=t))
    edits = [mix(0, scale=0.21), rot(0, base=510.0), kind(0, "latent_attention"), kind(1, "latent_attention_2"), kind(2, "latent_attention"), scl(1, factor=4.2), scl(1, original=80.0),
             scl(2, fast=3.0), scl(2, slow=5.0), lambda L: L[1]["mixer"]["rot"].pop("scaling"), lambda L: L[0].update(mlp=None)]
    for n, e in enumerate(edits):
        assert off(e) > 20 * F32_TOL, n
    for name in ("l0.norm1b", "l3.norm1b", "l0.norm2b", "l2.mix.sink", "l0.mlp.gate.b", "l0.mlp.up.b", "l0.mlp.down.b", "l1.mix.dq.norm", "l1.mix.dkv.norm"):
        w2 = dict(w)
        w2[name] = w[name] + 0.1
        assert rel(so.forward(cfg, w2, ids), full) > 20 * F32_TOL, name
    own = copy.deepcopy(cfg)
    del own["layers"][3]["mixer"]["kv_from"]
    w2 = dict(w, **{"l3.mix.dkv": w["l0.mix.dkv"], "l3.mix.dkv.norm": w["l0.mix.dkv.norm"]})
    assert rel(so.forward(own, w2, ids), full) > 20 * F32_TOL     # (the latents are layer 0's, not layer 0's matrix on layer 3's input)
