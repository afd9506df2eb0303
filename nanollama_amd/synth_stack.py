"""Random-weight model folders of layer-stack designs: there is no network for checkpoints, so tests and benchmarks write their own.

Matrices are normal with standard deviation gain / sqrt(inputs), norm gains near their neutral value, decay biases spread so that the
per-channel decays reach from nearly none to strong.  Values are drawn per tensor name: a tensor does not depend on the others."""
from __future__ import annotations

import json
import os
import zlib
from typing import Dict, Tuple

import numpy as np

from .safetensors import save, to_bf16


def ganidra_layer(kind: str, width_mlp: int = 0, **mixer) -> dict:
    return {"type": kind, "mixer": mixer, "mlp": {"kind": "dense", "ff": width_mlp} if width_mlp else None}


def ganidra_config(vocab: int, width: int, layers, loop=None, eps: float = 1e-5, embed_scale: float = 1.0) -> dict:
    cfg = {"architecture": "Ganidra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed_scale}, "layers": list(layers)}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def ganidra_shapes(cfg: dict, rank: int = 16) -> Dict[str, Tuple[int, ...]]:
    D = cfg["width"]
    out: Dict[str, Tuple[int, ...]] = {"embed": (cfg["vocab"], D)}

    def lin(p, m):
        H, k, v = m["heads"], m["dim"], m["vdim"]
        out.update({p + "q": (H * k, D), p + "k": (H * k, D), p + "v": (H * v, D), p + "g": (H * v, D), p + "o": (D, H * v), p + "norm": (v,),
                    p + "a1": (rank, D), p + "a2": (H * k, rank), p + "a2.b": (H * k,)})

    def attn(p, m):
        H, G, k, v = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out.update({p + "q": (H * k, D), p + "k": (G * k, D), p + "v": (G * v, D), p + "q.norm": (k,), p + "k.norm": (k,), p + "g": (H * v, D), p + "o": (D, H * v)})

    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        out[p + "norm1"] = (D,)
        if L["type"] == "gla":
            lin(p + "mix.", L["mixer"])
        else:
            attn(p + "mix.left.", L["mixer"]["left"])
            lin(p + "mix.right.", L["mixer"]["right"])
        if L["mlp"]:
            f = L["mlp"]["ff"]
            out.update({p + "norm2": (D,), p + "mlp.gate": (f, D), p + "mlp.up": (f, D), p + "mlp.down": (D, f)})
    out["final.norm"] = (D,)
    return out


def _fast_matrix(rng, shape, size: float) -> np.ndarray:
    n = shape[0] * shape[1]
    bits = rng.integers(0, 1 << 63, size=(n + 3) // 4, dtype=np.int64).view(np.uint16)[:n].reshape(shape)
    return (bits & np.uint16(0x807F)) | (np.uint16(127 + int(np.floor(np.log2(size)))) << np.uint16(7))


def ganidra_weights(cfg: dict, seed: int, rank: int = 16, gain: float = 1.0, fast: bool = False) -> Dict[str, np.ndarray]:
    """bfloat16 bits by tensor name.  fast: matrices are +- a constant with random mantissas (benchmarks of large models)."""
    out = {}
    for name, shape in ganidra_shapes(cfg, rank).items():
        rng = np.random.Generator(np.random.PCG64([seed, zlib.crc32(name.encode())]))
        if name == "final.norm" or name.endswith((".norm1", ".norm2")):
            x = 0.2 * rng.standard_normal(shape)           # gain 1 + w
        elif name.endswith(".norm"):
            x = 1.0 + 0.2 * rng.standard_normal(shape)
        elif name.endswith("a2.b"):
            x = rng.uniform(-3.0, 5.0, shape)
        elif len(shape) == 2 and fast and not name.endswith(("a1", "a2")):
            out[name] = _fast_matrix(rng, shape, gain / np.sqrt(shape[1] if name != "embed" else 1.0))
            continue
        else:
            x = rng.standard_normal(shape) * (1.0 if name == "embed" else gain / np.sqrt(shape[1]))
        out[name] = to_bf16(x.astype(np.float32))
    return out


def pabalix_layer(kind: int, ff: int = 0, **mixer) -> dict:
    """kind 1, 2 or 3; mixer: heads, dim, rot_dim, vdim, kv_rank, q_rank, base, scale (default 1 / sqrt(dim + rot_dim)), yarn (factor,
    original, fast, slow) or None, kv_from."""
    m = {k: mixer[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank")}
    m["scale"] = mixer.get("scale") or (m["dim"] + m["rot_dim"]) ** -0.5
    m["rot"] = {"base": float(mixer["base"]), "dims": m["rot_dim"]}
    if mixer.get("yarn"):
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), mixer["yarn"]))
    if mixer.get("kv_from") is not None:
        m["kv_from"] = mixer["kv_from"]
    return {"type": "latent_attention" + ("" if kind == 1 else f"_{kind}"), "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def pabalix_config(vocab: int, width: int, layers, eps: float = 1e-5) -> dict:
    return {"architecture": "Pabalix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": list(layers)}


def pabalix_shapes(cfg: dict) -> Dict[str, Tuple[int, ...]]:
    D = cfg["width"]
    out: Dict[str, Tuple[int, ...]] = {"embed": (cfg["vocab"], D), "final.norm": (D,), "head": (cfg["vocab"], D)}
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], f"l{i}.mix."
        H, q, kv = m["heads"], m["q_rank"], m["kv_rank"]
        out.update({f"l{i}.norm1": (D,), f"l{i}.norm1b": (D,), p + "dq": (q, D), p + "dq.norm": (q,), p + "uq": (H * (m["dim"] + m["rot_dim"]), q),
                    p + "uk": (H * m["dim"], kv), p + "uv": (H * m["vdim"], kv), p + "o": (D, H * m["vdim"])})
        if m.get("kv_from") is None:
            out.update({p + "dkv": (kv + m["rot_dim"], D), p + "dkv.norm": (kv,)})
        if L["type"].endswith("3"):
            out.update({p + "sink": (H,), p + "g": (H, D)})
        if L["mlp"]:
            f, p = L["mlp"]["ff"], f"l{i}.mlp."
            out.update({f"l{i}.norm2": (D,), f"l{i}.norm2b": (D,), p + "gate": (f, D), p + "gate.b": (f,), p + "up": (f, D), p + "up.b": (f,), p + "down": (D, f), p + "down.b": (D,)})
    return out


def pabalix_weights(cfg: dict, seed: int, gain: float = 1.0, fast: bool = False) -> Dict[str, np.ndarray]:
    """bfloat16 bits by tensor name; fast as in ganidra_weights."""
    out = {}
    for name, shape in pabalix_shapes(cfg).items():
        rng = np.random.Generator(np.random.PCG64([seed, zlib.crc32(name.encode())]))
        if len(shape) == 2 and fast:
            out[name] = _fast_matrix(rng, shape, 1.0 if name == "embed" else gain / np.sqrt(max(1, shape[1])))
            continue
        if len(shape) == 2:
            x = rng.standard_normal(shape) * (1.0 if name == "embed" else gain / np.sqrt(max(1, shape[1])))
        elif "norm" in name:
            x = 1.0 + 0.2 * rng.standard_normal(shape)
        elif name.endswith("sink"):
            x = rng.uniform(-1.0, 3.0, shape)
        else:
            x = 0.3 * rng.standard_normal(shape)               # biases
        out[name] = to_bf16(x.astype(np.float32))
    return out


def write_folder(path: str, cfg: dict, weights: Dict[str, np.ndarray]) -> str:
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f, indent=1)
    save(os.path.join(path, "model.safetensors"), weights)
    return path
