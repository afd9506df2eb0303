"""Models described layer by layer over libnanollama_stack.so (include/nanollama_stack.h).

A design (nanollama_amd/designs/) turns its config.json and tensor names into a StackSpec; load_stack_model hands the weights to
the device library and returns a StackModel, which the generation loop, the batch scheduler, the CLI and the server use like any
other HipModel.  All arithmetic happens in the library.
"""
from __future__ import annotations

import ctypes as C
from dataclasses import dataclass, field
from typing import Callable, Dict, List, Optional, Tuple

import numpy as np

from . import _lib
from .model import HipModel

DTYPES = {"bfloat16": 0, "float32": 1}
DEFAULT_SEQ_LEN = 8192          # these designs carry no limit of their own: positions per stream a model is loaded for


@dataclass
class Attention:
    """Softmax attention, see nl_attn_desc."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int = 0
    qk_norm: bool = False
    distance_bias: bool = False
    gate: bool = False
    mix_scale: float = 1.0


@dataclass
class LinearAttention:
    """Gated linear attention with a decay per key channel, see nl_linattn_desc."""
    heads: int
    dim: int
    vdim: int
    rank: int
    tau: float
    mix_scale: float = 1.0


@dataclass
class Yarn:
    """Interpolated rotary frequencies."""
    factor: float
    original: float
    fast: float
    slow: float


@dataclass
class LatentAttention:
    """Softmax attention over keys and values that are images of one cached latent, see nl_latent_desc."""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rope_base: float
    rot_dims: int
    adjacent_pairs: bool = False
    yarn: Optional[Yarn] = None
    kv_from: Optional[int] = None
    sink: bool = False
    gate: bool = False


ACTIVATIONS = {"gelu_tanh": 0, "silu": 1}


@dataclass
class StackLayer:
    attn: Optional[Attention] = None
    lin: Optional[LinearAttention] = None
    latent: Optional[LatentAttention] = None
    ff: int = 0
    ff_act: str = "gelu_tanh"
    ff_bias: bool = False

    def mixers(self):
        return [m for m in (self.attn, self.lin, self.latent) if m]


@dataclass
class StackSpec:
    architecture: str
    vocab: int
    dim: int
    layers: List[StackLayer]
    eps: float
    embed_scale: float = 1.0
    loop: Optional[Tuple[int, int, int]] = None      # start, stop, times
    plain_norm: bool = False                         # norm gains are w, not 1 + w
    post_norm: bool = False                          # a norm behind every sublayer
    untied: bool = False                             # an output matrix of its own
    tensors: Dict[str, str] = field(default_factory=dict)   # library name -> name in the weight file

    def runs(self) -> List[int]:
        """Layers in the order they are executed."""
        n = len(self.layers)
        if not self.loop:
            return list(range(n))
        a, b, k = self.loop
        return list(range(a)) + list(range(a, b)) * k + list(range(b, n))


class StackConfig:
    """What the host layers ask a model's configuration for (the names of LlamaConfig)."""

    def __init__(self, spec: StackSpec, seq_len: int, dtype: str, num_params: int):
        self.spec, self.seq_len, self.dtype, self.num_params = spec, seq_len, dtype, num_params
        self.architecture = spec.architecture
        self.num_layers, self.embed_dim, self.vocab_size = len(spec.layers), spec.dim, spec.vocab
        self.num_heads = max(m.heads for l in spec.layers for m in l.mixers())
        self.num_kv_heads = max((l.attn.kv_heads for l in spec.layers if l.attn), default=0)
        self.interm_size = max(l.ff for l in spec.layers)
        self.rms_norm_eps = spec.eps
        self.qk_norm = any(l.attn and l.attn.qk_norm for l in spec.layers)
        self.rope_conjugate = False


class StackModel(HipModel):
    def __init__(self, config: StackConfig, handle, max_streams: int):
        super().__init__(config, handle, max_streams, _lib.stack_lib())

    def step(self, entries):
        """HipModel.step as ONE ragged launch sequence (nl_step)."""
        n = len(entries)
        toks = [int(t) for e in entries for t in e[1]]
        ia = lambda v: (C.c_int * max(len(v), 1))(*v)
        want, at = [], 0
        for _, tokens, _, w in entries:
            want += [at + int(k) for k in sorted(set(w))]
            at += len(tokens)
        lg = np.zeros((len(want), self.config.vocab_size), np.float32)
        self._check(self._L.nl_step(self._h, n, ia([int(e[0]) for e in entries]), ia([len(e[1]) for e in entries]), ia([int(e[2]) for e in entries]),
                                    ia(toks), len(want), ia(want), lg.ctypes.data_as(C.POINTER(C.c_float)), None))
        out, at = [], 0
        for _, _, _, w in entries:
            order = {k: i for i, k in enumerate(sorted(set(w)))}
            out.append(lg[[at + order[k] for k in w]] if len(w) else lg[:0])
            at += len(order)
        return out

    def trace_layers(self, on: bool = True) -> None:
        """Keep the residual stream behind every layer run (layer_trace reads it); graph replay is off meanwhile."""
        self._check(self._L.nl_trace_layers(self._h, int(on)))

    def layer_trace(self, n_tokens: int) -> np.ndarray:
        """[layer runs, tokens of the last launch sequence, width]"""
        runs, d = len(self.config.spec.runs()), self.config.embed_dim
        return self.debug_read("layers", runs * n_tokens * d).reshape(runs, n_tokens, d)


def _layer_desc(layer: StackLayer) -> _lib.NlLayerDesc:
    d = _lib.NlLayerDesc()
    if layer.attn:
        a = layer.attn
        d.attn = _lib.NlAttnDesc(a.heads, a.kv_heads, a.dim, a.vdim, a.window, int(a.qk_norm), int(a.distance_bias), int(a.gate), a.scale, a.mix_scale)
    if layer.lin:
        g = layer.lin
        d.lin = _lib.NlLinattnDesc(g.heads, g.dim, g.vdim, g.rank, g.tau, g.mix_scale)
    if layer.latent:
        t, y = layer.latent, layer.latent.yarn or Yarn(0.0, 0.0, 0.0, 0.0)
        d.latent = _lib.NlLatentDesc(t.heads, t.dim, t.rot_dim, t.vdim, t.q_rank, t.kv_rank, -1 if t.kv_from is None else t.kv_from, t.rot_dims,
                                     int(t.adjacent_pairs), int(t.sink), int(t.gate), t.scale, t.rope_base, y.factor, y.original, y.fast, y.slow)
    d.ff, d.ff_act, d.ff_bias = layer.ff, ACTIVATIONS[layer.ff_act], int(layer.ff_bias)
    return d


def load_stack_model(spec: StackSpec, get: Callable[[str], Tuple[str, np.ndarray]], device: int = 0, max_streams: int = 1,
                     seq_len: int = 0, dtype: str = "bfloat16", max_step_tokens: int = 0, flags: int = 0, verbose: bool = False) -> StackModel:
    """get(name in the weight file) -> (dtype tag, array), as SafetensorsFile.get."""
    if dtype not in DTYPES:
        raise ValueError(f"dtype {dtype!r}: one of {', '.join(DTYPES)}")
    L = _lib.stack_lib()
    seq_len = seq_len or DEFAULT_SEQ_LEN
    start, stop, times = spec.loop or (0, 0, 1)
    cfg = _lib.NlStackConfig(spec.vocab, spec.dim, len(spec.layers), start, stop, times, seq_len, max_streams, max_step_tokens, device,
                             DTYPES[dtype], flags, int(spec.plain_norm), int(spec.post_norm), int(spec.untied), spec.eps, spec.embed_scale)
    descs = (_lib.NlLayerDesc * len(spec.layers))(*[_layer_desc(l) for l in spec.layers])
    h = C.c_void_p()
    rc = L.nl_create_stack(C.byref(cfg), descs, C.byref(h))
    if rc != 0:
        raise _lib.NlError(rc, (L.nl_last_error(None) or b"").decode())
    params = 0
    try:
        for name, source in spec.tensors.items():
            tag, x = get(source)
            if tag not in ("F32", "BF16"):
                raise ValueError(f"tensor {source}: type {tag} (float32 and bfloat16 are taken)")
            x = np.ascontiguousarray(x)
            rows, cols = (1, x.shape[0]) if x.ndim == 1 else x.shape
            params += x.size
            _lib.check(h, L.nl_upload_tensor(h, name.encode(), 0 if tag == "F32" else 30, x.ctypes.data, x.nbytes, rows, cols), L)
        _lib.check(h, L.nl_finalize(h), L)
    except Exception:
        L.nl_destroy(h)
        raise
    config = StackConfig(spec, seq_len, dtype, params)
    if verbose:
        print(f"[model] loaded: {spec.architecture}, {len(spec.layers)} layers ({len(spec.runs())} runs), {spec.dim} dim, {spec.vocab} vocab, {dtype}")
    return StackModel(config, h, max_streams)
