"""Plain float64 restatement of the layer-stack models (Ganidra, Pabalix), one function per mechanism, whole sequences, no cache.

TEST INFRASTRUCTURE ONLY -- importable from tests/, never from nanollama_amd/; it shares no code with the product.
`cfg` is the dictionary of config.json, `w` a dictionary of float arrays by tensor name (matrices [out, in]).
"""
from __future__ import annotations

import numpy as np


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm_one_plus(x, weight, eps):
    """The residual stream's norm: gain 1 + weight."""
    return rms(x, eps) * (1.0 + weight)


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def log_sigmoid(z):
    return np.minimum(z, 0.0) - np.log1p(np.exp(-np.abs(z)))


def key_decay(h, a1, a2, bias, tau):
    """Per-channel decay alpha = sigmoid(a2 (a1 h) + bias)^(1 / tau), [T, heads * dim]."""
    return np.exp(log_sigmoid(h @ a1.T @ a2.T + bias) / tau)


def gated_recurrence(q, k, v, alpha, state=None):
    """S_t = diag(alpha_t) S_{t-1} + k_t v_t^T, o_t = S_t^T q_t for one head.  q, k, alpha [T, dk]; v [T, dv].
    Returns (o [T, dv], last state [dk, dv])."""
    S = np.zeros((q.shape[1], v.shape[1])) if state is None else state.copy()
    out = np.zeros_like(v)
    for t in range(q.shape[0]):
        S = alpha[t][:, None] * S + np.outer(k[t], v[t])
        out[t] = S.T @ q[t]
    return out, S


def gla_mixer(h, m, w, p, eps):
    """Gated linear attention; m = the mixer's entry, p = the tensors' prefix."""
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ w[p + "q"].T).reshape(T, H, dk) * dk ** -0.5
    k = (h @ w[p + "k"].T).reshape(T, H, dk)
    v = (h @ w[p + "v"].T).reshape(T, H, dv)
    alpha = key_decay(h, w[p + "a1"], w[p + "a2"], w[p + "a2.b"], m["tau"]).reshape(T, H, dk)
    o = np.stack([gated_recurrence(q[:, j], k[:, j], v[:, j], alpha[:, j])[0] for j in range(H)], axis=1)
    o = rms(o, eps) * w[p + "norm"]
    return (o.reshape(T, H * dv) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def attention_weights(q, k, scale, slope, window):
    """Softmax weights of one head: (q . k) * scale - slope * (i - j) over the keys i - window < j <= i."""
    T = q.shape[0]
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    s = (q @ k.T) * scale - slope * (i - j)
    seen = (j <= i) if window is None else (j <= i) & (i - j < window)
    s = np.where(seen, s, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def window_attention(h, m, w, p, eps):
    """Grouped-query attention with per-head query / key norm, a linear distance bias, a sliding window and an output gate."""
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = rms((h @ w[p + "q"].T).reshape(T, H, dk), eps) * w[p + "q.norm"]
    k = rms((h @ w[p + "k"].T).reshape(T, G, dk), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T).reshape(T, G, dv)
    window = m["mask"]["size"] if m.get("mask") else None
    out = np.zeros((T, H, dv))
    for a in range(H):
        g = a // (H // G)
        out[:, a] = attention_weights(q[:, a], k[:, g], m["scale"], 2.0 ** (-8.0 * (a + 1) / H), window) @ v[:, g]
    return (out.reshape(T, H * dv) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel_mixer(h, m, w, p, eps):
    return m["left_scale"] * window_attention(h, m["left"], w, p + "left.", eps) + \
        m["right_scale"] * gla_mixer(h, m["right"], w, p + "right.", eps)


MIXERS = {"gla": gla_mixer, "parallel": parallel_mixer}


def gated_mlp(h, w, p):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def layer_runs(cfg):
    """[(layer, add the embedding output first?)] in execution order."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b, k = loop["start"], loop["stop"], loop["times"]
    runs = [(i, False) for i in range(a)]
    for t in range(k):
        runs += [(i, t > 0 and i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


# ---- latent attention (Pabalix) -------------------------------------------------------------------------------------------------

def norm_plain(x, weight, eps):
    return rms(x, eps) * weight


def rotary_frequencies(rot):
    """(angle per position for each pair, factor of cos and sin); rot: dims, base and, for YaRN, scaling."""
    n, base = rot["dims"], float(rot["base"])
    f = base ** (-2.0 * np.arange(n // 2) / n)
    y = rot.get("scaling")
    if not y:
        return f, 1.0
    turns = lambda t: n * np.log(y["original"] / (2 * np.pi * t)) / (2 * np.log(base))    # the pair that turns t times over `original`
    lo, hi = max(np.floor(turns(y["fast"])), 0.0), min(np.ceil(turns(y["slow"])), n - 1.0)
    slow = np.clip((np.arange(n // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / y["factor"] * slow + f * (1.0 - slow), 0.1 * np.log(y["factor"]) + 1.0


def rotate(x, rot, interleaved):
    """x [T, ..., rot_dim], row t at position t."""
    f, m = rotary_frequencies(rot)
    a = np.arange(x.shape[0])[:, None] * f
    shape = (x.shape[0],) + (1,) * (x.ndim - 2) + (len(f),)
    c, s = (m * np.cos(a)).reshape(shape), (m * np.sin(a)).reshape(shape)
    n = len(f)
    first, second = (slice(0, 2 * n, 2), slice(1, 2 * n, 2)) if interleaved else (slice(0, n), slice(n, 2 * n))
    out = x.copy()
    out[..., first] = x[..., first] * c - x[..., second] * s
    out[..., second] = x[..., second] * c + x[..., first] * s
    return out


def sink_softmax(s, sink=None):
    """Rows of scores with -inf for unseen keys; sink: a score of the denominator alone."""
    m = s.max(axis=-1, keepdims=True) if sink is None else np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.exp(s - m)
    return e / (e.sum(axis=-1, keepdims=True) + (0.0 if sink is None else np.exp(sink - m)))


LATENT_KINDS = {                 # type -> (adjacent dimensions are a pair, sink, gate per head)
    "latent_attention": (False, False, False),
    "latent_attention_2": (True, False, False),
    "latent_attention_3": (False, True, True),
}


def latent_keys(h, m, w, p, eps, interleaved):
    """(latent [T, kv_rank], rotated key part [T, rot_dim]): what a cache holds."""
    c = h @ w[p + "dkv"].T
    return norm_plain(c[:, :m["kv_rank"]], w[p + "dkv.norm"], eps), rotate(c[:, m["kv_rank"]:], m["rot"], interleaved)


def latent_attention(h, m, w, p, eps, kind, held):
    """held: latent_keys of this layer or of the layer that it borrows them from."""
    H, d, r, v = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    interleaved, sink, gate = LATENT_KINDS[kind]
    T = h.shape[0]
    q = (norm_plain(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).reshape(T, H, d + r)
    qr = rotate(q[..., d:], m["rot"], interleaved)
    c, kr = held
    k = (c @ w[p + "uk"].T).reshape(T, H, d)
    val = (c @ w[p + "uv"].T).reshape(T, H, v)
    seen = np.tril(np.ones((T, T), bool))
    out = np.zeros((T, H, v))
    for a in range(H):
        s = np.where(seen, (q[:, a, :d] @ k[:, a].T + qr[:, a] @ kr.T) * m["scale"], -np.inf)
        out[:, a] = sink_softmax(s, w[p + "sink"][a] if sink else None) @ val[:, a]
    if gate:
        out = out * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return out.reshape(T, H * v) @ w[p + "o"].T


def biased_silu_mlp(h, w, p):
    return (silu(h @ w[p + "gate"].T + w[p + "gate.b"]) * (h @ w[p + "up"].T + w[p + "up.b"])) @ w[p + "down"].T + w[p + "down.b"]


def latent_forward(cfg, w, tokens, want_layers=False):
    """Pabalix: norms in front of and behind every sublayer, latent attention, an output matrix of its own."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)]
    seen, held = [], {}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        h = norm_plain(x, w[p + "norm1"], eps)
        if m.get("kv_from") is None:
            held[i] = latent_keys(h, m, w, p + "mix.", eps, LATENT_KINDS[L["type"]][0])
        o = latent_attention(h, m, w, p + "mix.", eps, L["type"], held[i if m.get("kv_from") is None else m["kv_from"]])
        x = x + norm_plain(o, w[p + "norm1b"], eps)
        if L["mlp"] is not None:
            x = x + norm_plain(biased_silu_mlp(norm_plain(x, w[p + "norm2"], eps), w, p + "mlp."), w[p + "norm2b"], eps)
        seen.append(x)
    logits = norm_plain(x, w["final.norm"], eps) @ w["head"].T
    return (logits, np.stack(seen)) if want_layers else logits


def forward(cfg, w, tokens, want_layers=False):
    """Logits [T, vocab] (and the residual stream after every layer run)."""
    if cfg["architecture"] == "Pabalix":
        return latent_forward(cfg, w, tokens, want_layers)
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    x0 = x.copy()
    seen = []
    for i, add in layer_runs(cfg):
        if add:
            x = x + x0
        L, p = cfg["layers"][i], f"l{i}."
        x = x + MIXERS[L["type"]](norm_one_plus(x, w[p + "norm1"], eps), L["mixer"], w, p + "mix.", eps)
        if L["mlp"] is not None:
            x = x + gated_mlp(norm_one_plus(x, w[p + "norm2"], eps), w, p + "mlp.")
        seen.append(x)
    logits = norm_one_plus(x, w["final.norm"], eps) @ w["embed"].T
    return (logits, np.stack(seen)) if want_layers else logits


def greedy(cfg, w, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(np.argmax(forward(cfg, w, ids)[-1])))
    return ids[len(prompt):]
