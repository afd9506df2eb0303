"""Pabalix: latent attention in every layer (three kinds: rotary pairs half a vector apart with YaRN, adjacent pairs where a layer may
attend an earlier layer's latents, and the first kind with a sink and a gate per head), norms in front of and behind every sublayer, an
optional silu feed-forward with biases, an output matrix of its own."""
from __future__ import annotations

from typing import Callable, Tuple

from ..stack import LatentAttention, StackLayer, StackSpec, Yarn

# type of a mixer -> (adjacent dimensions are a rotary pair, sink and gate per head)
KINDS = {"latent_attention": (False, False), "latent_attention_2": (True, False), "latent_attention_3": (False, True)}


def pabalix_spec(cfg: dict, shape: Callable[[str], Tuple[int, ...]]) -> StackSpec:
    tensors = {"embed": "embed", "head": "head", "final_norm": "final.norm"}
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        kind, m, mlp = entry["type"], entry["mixer"], entry.get("mlp")
        if kind not in KINDS:
            raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
        adjacent, sink_gate = KINDS[kind]
        rot, held = m["rot"], m.get("kv_from")
        y = rot.get("scaling")
        layer = StackLayer(latent=LatentAttention(
            m["heads"], m["dim"], m["rot_dim"], m["vdim"], shape(f"l{i}.mix.dq")[0], m["kv_rank"], m["scale"], rot["base"], rot["dims"], adjacent,
            Yarn(y["factor"], y["original"], y["fast"], y["slow"]) if y else None, held, sink_gate, sink_gate))
        names = {"dq": "dq", "q_norm": "dq.norm", "uq": "uq", "uk": "uk", "uv": "uv", "o": "o"}
        if held is None:
            names.update(dkv="dkv", kv_norm="dkv.norm")
        if sink_gate:
            names.update(sink="sink", g="g")
        tensors.update({f"layers.{i}.latent.{k}": f"l{i}.mix.{v}" for k, v in names.items()})
        tensors.update({f"layers.{i}.norm1": f"l{i}.norm1", f"layers.{i}.norm1_post": f"l{i}.norm1b"})
        if mlp is not None:
            if mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
            layer.ff, layer.ff_act, layer.ff_bias = mlp["ff"], "silu", True
            tensors.update({f"layers.{i}.norm2": f"l{i}.norm2", f"layers.{i}.norm2_post": f"l{i}.norm2b"})
            for k in ("gate", "up", "down"):
                tensors.update({f"layers.{i}.ff.{k}": f"l{i}.mlp.{k}", f"layers.{i}.ff.{k}_bias": f"l{i}.mlp.{k}.b"})
        layers.append(layer)
    return StackSpec("Pabalix", cfg["vocab"], cfg["width"], layers, cfg["norm"]["eps"], plain_norm=True, post_norm=True, untied=True, tensors=tensors)
