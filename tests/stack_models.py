"""Small layer-stack models for the tests: configurations, random weights, loading, and the error measure."""
import numpy as np

from nanollama_amd import synth_stack as ss
from nanollama_amd.safetensors import from_bf16, to_bf16

F32_TOL, BF16_TOL = 4e-5, 5e-2


def gla(heads=2, dim=16, vdim=16, tau=8.0, ff=0):
    return ss.ganidra_layer("gla", ff, heads=heads, dim=dim, vdim=vdim, tau=tau)


def par(heads=2, kv=1, dim=32, vdim=32, window=24, scale=None, rheads=2, rdim=16, rvdim=16, tau=8.0, ls=0.7, rs=1.3, ff=0):
    left = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5}
    if window:
        left["mask"] = {"size": window}
    return ss.ganidra_layer("parallel", ff, left=left, right={"heads": rheads, "dim": rdim, "vdim": rvdim, "tau": tau}, left_scale=ls, right_scale=rs)


def config(layers, vocab=96, width=64, loop=None, eps=1e-5, embed_scale=1.5):
    return ss.ganidra_config(vocab, width, layers, loop, eps, embed_scale)


def lat(kind=1, heads=3, dim=16, rot=8, vdim=16, kv_rank=32, q_rank=24, base=500.0, scale=None, yarn=None, kv_from=None, ff=0):
    return ss.pabalix_layer(kind, ff, heads=heads, dim=dim, rot_dim=rot, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, base=base, scale=scale, yarn=yarn, kv_from=kv_from)


def lconfig(layers, vocab=96, width=64, eps=1e-5):
    return ss.pabalix_config(vocab, width, layers, eps)


def weights(cfg, seed=1, rank=4):
    return ss.pabalix_weights(cfg, seed) if cfg["architecture"] == "Pabalix" else ss.ganidra_weights(cfg, seed, rank)


def floats(w):
    """bfloat16 bits -> what the oracle computes with."""
    return {k: from_bf16(v).astype(np.float64).reshape(v.shape) for k, v in w.items()}


def bits(w):
    return {k: to_bf16(v.astype(np.float32)).reshape(v.shape) for k, v in w.items()}


def load(cfg, w, dtype="float32", max_streams=4, seq_len=512, max_step_tokens=0, flags=0):
    from nanollama_amd.designs import DESIGNS
    from nanollama_amd.stack import load_stack_model
    spec = DESIGNS[cfg["architecture"]](cfg, lambda n: w[n].shape)
    return load_stack_model(spec, lambda n: ("BF16", w[n]), 0, max_streams, seq_len, dtype, max_step_tokens, flags)


def tokens(n, vocab=96, seed=0):
    return [int(t) for t in np.random.default_rng(seed).integers(0, vocab, n)]


def rel(got, want):
    """Largest over the rows: rms difference over the vocabulary / spread of the logits."""
    got, want = np.atleast_2d(np.asarray(got, np.float64)), np.atleast_2d(want)
    return float(np.max(np.sqrt(np.mean((got - want) ** 2, axis=-1))) / np.std(want))
