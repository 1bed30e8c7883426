"""Plain, slow restatement of the Ligidra design on the CPU (test infrastructure only; shares no code with the product path
under nano_vllm_amd/). One function per mechanism, float64 throughout, loops over tokens wherever the design has a
recurrence, a convolution over time or a mask.

The design: a pre-norm decoder whose layers are listed one by one. The embedding row is normed; every mixer reads its normed
input blended, channel by channel, with the previous token's; after the feed-forward a third branch adds a normed projection of
(a gated part of a second embedding table). Mixers: `attention` (q / k norms over the whole projection, rotation in interleaved
pairs with band-wise scaled frequencies, capped scores, a learned sink, a sliding window whose past is kept as means over blocks
of positions; a layer may read the keys and values of an earlier one), `delta` and `channel_delta` (the gated delta rule with a
decay per head, or per head and key channel). Feed-forward: softmax-routed gated experts beside a shared one.
"""
from __future__ import annotations

import math

import numpy as np


def f64(t) -> np.ndarray:
    import torch
    if isinstance(t, torch.Tensor):
        return t.to(torch.float64).numpy() if t.is_floating_point() else t.numpy().astype(np.int64)
    return np.asarray(t)


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_tanh(z: np.ndarray) -> np.ndarray:
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def norm(x: np.ndarray, w, eps: float) -> np.ndarray:
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def token_shift(h: np.ndarray, mu: np.ndarray) -> np.ndarray:
    """h [T, W] blended with the row before it (zeros before the first)."""
    before = np.zeros_like(h)
    before[1:] = h[:-1]
    return h + (before - h) * mu


def token_side(x: np.ndarray, e: np.ndarray, w: dict, eps: float) -> np.ndarray:
    g = gelu_tanh(x @ w["gate"].T) * e
    return norm(g @ w["proj"].T, w["norm"], eps)


def frequencies(rot: dict) -> np.ndarray:
    dims, base = int(rot["dims"]), float(rot["base"])
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=np.float64)
    sc = rot.get("scaling")
    if not sc:
        return f
    factor, low, high, orig = float(sc["factor"]), float(sc["low"]), float(sc["high"]), float(sc["original"])
    out = f.copy()
    for i, fi in enumerate(f):
        length = 2.0 * math.pi / fi
        if length < orig / high:
            continue
        if length > orig / low:
            out[i] = fi / factor
        else:
            s = (orig / length - low) / (high - low)
            out[i] = (1.0 - s) * fi / factor + s * fi
    return out


def rotate_pairs(x: np.ndarray, freq: np.ndarray) -> np.ndarray:
    """x [T, heads, d], row t at position t: entries (2i, 2i+1), i < len(freq), turn by t * freq[i]; the rest pass."""
    out = x.copy()
    pos = np.arange(x.shape[0], dtype=np.float64)
    for i, fi in enumerate(freq):
        c, s = np.cos(pos * fi)[:, None], np.sin(pos * fi)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def pooled_attention(q: np.ndarray, k: np.ndarray, v: np.ndarray, scale: float, cap: float, sink: np.ndarray, size: int, pool: int) -> np.ndarray:
    """q [T, H, d], k [T, G, d], v [T, G, dv]. Row t sees the last `size` rows, and one mean key / value for every block of `pool`
    rows all of which lie before those; score = cap tanh(q.k scale / cap); the denominator also holds exp(sink[head])."""
    T, H, _ = q.shape
    G, dv = v.shape[1], v.shape[2]
    out = np.zeros((T, H, dv))
    for t in range(T):
        seen_k, seen_v = [], []
        b = 0
        while b * pool + pool - 1 <= t - size:
            seen_k.append(k[b * pool:(b + 1) * pool].mean(0))
            seen_v.append(v[b * pool:(b + 1) * pool].mean(0))
            b += 1
        for j in range(max(0, t - size + 1), t + 1):
            seen_k.append(k[j])
            seen_v.append(v[j])
        ks, vs = np.stack(seen_k), np.stack(seen_v)
        for a in range(H):
            g = a // (H // G)
            s = (ks[:, g] @ q[t, a]) * scale
            if cap:
                s = cap * np.tanh(s / cap)
            m = max(s.max(), sink[a])
            e = np.exp(s - m)
            out[t, a] = (e @ vs[:, g]) / (e.sum() + math.exp(sink[a] - m))
    return out


def attention(h: np.ndarray, w: dict, m: dict, eps: float, kv: tuple | None = None):
    """(output, (keys, values)); `kv`: the keys (normed and rotated) and values of another layer to use instead of own ones."""
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    rot = m.get("rot")
    q = norm(h @ w["q"].T, w["q.norm"], eps).reshape(T, H, d)
    if rot:
        q = rotate_pairs(q, frequencies(rot))
    if kv is None:
        k = norm(h @ w["k"].T, w["k.norm"], eps).reshape(T, G, d)
        if rot:
            k = rotate_pairs(k, frequencies(rot))
        kv = (k, (h @ w["v"].T).reshape(T, G, dv))
    mask = m.get("mask")
    size, pool = (int(mask["size"]), int(mask["pool"])) if mask else (T, T + 1)
    o = pooled_attention(q, kv[0], kv[1], float(m["scale"]), float(m.get("softcap") or 0.0), w["sink"], size, pool)
    return o.reshape(T, -1) @ w["o"].T, kv


def short_conv(u: np.ndarray, w: np.ndarray) -> np.ndarray:
    """u [T, C], w [C, taps]: y_t = silu(sum_j w[:, j] u_(t - taps + 1 + j)), zeros before the first token."""
    T, taps = u.shape[0], w.shape[1]
    y = np.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            src = t - taps + 1 + j
            if src >= 0:
                y[t] += w[:, j] * u[src]
    return silu(y)


def unit(x: np.ndarray) -> np.ndarray:
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def delta_rule(q: np.ndarray, k: np.ndarray, v: np.ndarray, beta: np.ndarray, decay: np.ndarray) -> np.ndarray:
    """One head: q, k [T, d], v [T, dv], beta [T], decay [T] or [T, d] (then it acts on the rows of the state)."""
    T, d = k.shape
    S = np.zeros((d, v.shape[1]))
    out = np.zeros_like(v)
    for t in range(T):
        S = (decay[t] * np.ones(d))[:, None] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + np.outer(k[t], u)
        out[t] = S.T @ q[t]
    return out


def delta(h: np.ndarray, w: dict, m: dict, eps: float, per_channel: bool) -> np.ndarray:
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = unit(short_conv(h @ w["q"].T, w["q.conv"]).reshape(T, G, d)) * d ** -0.5
    k = unit(short_conv(h @ w["k"].T, w["k.conv"]).reshape(T, G, d))
    v = short_conv(h @ w["v"].T, w["v.conv"]).reshape(T, H, dv)
    beta = sigmoid(h @ w["b"].T)
    rate = np.exp(w["A_log"])
    if per_channel:
        z = ((h @ w["a1"].T) @ w["a2"].T + w["dt_bias"]).reshape(T, H, d)
        decay = np.exp(-rate[:, None] * softplus(z))
        gate = sigmoid((h @ w["g1"].T) @ w["g2"].T)
    else:
        decay = np.exp(-rate * softplus(h @ w["a"].T + w["dt_bias"]))
        gate = silu(h @ w["g"].T)
    o = np.zeros((T, H, dv))
    for a in range(H):
        g = a // (H // G)
        o[:, a] = delta_rule(q[:, g], k[:, g], v[:, a], beta[:, a], decay[:, a])
    return (norm(o, w["norm"], eps).reshape(T, -1) * gate) @ w["o"].T


def gated_unit(h: np.ndarray, w: dict) -> np.ndarray:
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def _sub(tensors: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def experts(h: np.ndarray, w: dict, mlp: dict) -> np.ndarray:
    z = h @ w["router"].T
    e = np.exp(z - z.max(-1, keepdims=True))
    s = e / e.sum(-1, keepdims=True)
    out = np.zeros_like(h)
    units = [_sub(w, f"e{i}.") for i in range(int(mlp["router"]["experts"]))]
    for t in range(h.shape[0]):
        for i in np.argsort(-s[t], kind="stable")[:int(mlp["router"]["top"])]:
            out[t] += s[t, i] * gated_unit(h[t:t + 1], units[int(i)])[0]
    if mlp.get("shared"):
        out = out + gated_unit(h, _sub(w, "shared."))
    return out


def forward(raw: dict, tensors: dict, tokens, trace: list | None = None) -> np.ndarray:
    """Logits [T, vocab] of one sequence; `trace` receives the residual rows after every layer."""
    eps = float(raw["norm"]["eps"])
    tokens = np.asarray(tokens)
    x = norm(tensors["embed"][tokens], tensors["embed.norm"], eps)
    cached = {}
    for i, layer in enumerate(raw["layers"]):
        w, m = _sub(tensors, f"l{i}."), layer["mixer"]
        h = token_shift(norm(x, w["norm1"], eps), w["shift"])
        wm = _sub(w, "mix.")
        if layer["type"] == "attention":
            y, cached[i] = attention(h, wm, m, eps, cached[int(m["kv_from"])] if m.get("kv_from") is not None else None)
        else:
            assert layer["type"] in ("delta", "channel_delta")
            y = delta(h, wm, m, eps, layer["type"] == "channel_delta")
        x = x + y
        if layer.get("mlp") is not None:
            x = x + experts(norm(x, w["norm2"], eps), _sub(w, "mlp."), layer["mlp"])
        if raw.get("token_side"):
            n = int(raw["token_side"]["dim"])
            x = x + token_side(x, tensors["side.embed"][tokens][:, i * n:(i + 1) * n], _sub(w, "side."), eps)
        if trace is not None:
            trace.append(x.copy())
    return norm(x, tensors["final.norm"], eps) @ tensors["embed"].T


class Model:
    """A checkpoint (configuration + tensors) read into float64."""

    def __init__(self, cfg: dict, tensors: dict):
        self.cfg, self.tensors = cfg, {k: f64(v) for k, v in tensors.items()}

    @classmethod
    def load(cls, path: str) -> "Model":
        import json
        import os

        from safetensors.torch import load_file
        with open(os.path.join(path, "config.json")) as fh:
            cfg = json.load(fh)
        return cls(cfg, load_file(os.path.join(path, "model.safetensors")))

    def run(self, tokens, trace: list | None = None) -> np.ndarray:
        return forward(self.cfg, self.tensors, tokens, trace)
