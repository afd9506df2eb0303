"""Ganidra: gated linear attention layers ("gla") and layers whose mixer runs windowed softmax attention and gated linear attention
side by side ("parallel"), an optional gated feed-forward per layer, a range of layers that is run several times, tied output."""
from __future__ import annotations

from typing import Callable, Tuple

from ..stack import Attention, LinearAttention, StackLayer, StackSpec

_LIN = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "a1": "a1", "a2": "a2", "a2_bias": "a2.b", "norm": "norm"}
_ATTN = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm"}


def ganidra_spec(cfg: dict, shape: Callable[[str], Tuple[int, ...]]) -> StackSpec:
    tensors = {"embed": "embed", "final_norm": "final.norm"}

    def lin(i: int, m: dict, prefix: str, scale: float) -> LinearAttention:
        tensors.update({f"layers.{i}.lin.{k}": prefix + v for k, v in _LIN.items()})
        return LinearAttention(m["heads"], m["dim"], m["vdim"], shape(prefix + "a1")[0], m["tau"], scale)

    def attn(i: int, m: dict, prefix: str, scale: float) -> Attention:
        tensors.update({f"layers.{i}.attn.{k}": prefix + v for k, v in _ATTN.items()})
        mask = m.get("mask") or {}
        return Attention(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], window=mask.get("size", 0), qk_norm=True,
                         distance_bias=True, gate=True, mix_scale=scale)

    layers = []
    for i, entry in enumerate(cfg["layers"]):
        kind, m, mlp = entry["type"], entry["mixer"], entry.get("mlp")
        layer = StackLayer()
        tensors[f"layers.{i}.norm1"] = f"l{i}.norm1"
        if kind == "gla":
            layer.lin = lin(i, m, f"l{i}.mix.", 1.0)
        elif kind == "parallel":
            layer.attn = attn(i, m["left"], f"l{i}.mix.left.", m["left_scale"])
            layer.lin = lin(i, m["right"], f"l{i}.mix.right.", m["right_scale"])
        else:
            raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
        if mlp is not None:
            if mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
            layer.ff = mlp["ff"]
            tensors[f"layers.{i}.norm2"] = f"l{i}.norm2"
            tensors.update({f"layers.{i}.ff.{k}": f"l{i}.mlp.{k}" for k in ("gate", "up", "down")})
        layers.append(layer)
    loop = cfg.get("loop")
    return StackSpec("Ganidra", cfg["vocab"], cfg["width"], layers, cfg["norm"]["eps"], cfg["embedding"]["scale"],
                     (loop["start"], loop["stop"], loop["times"]) if loop else None, tensors=tensors)
