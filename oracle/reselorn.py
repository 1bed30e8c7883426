"""Plain, slow restatement of the Reselorn design on the CPU (test infrastructure only; shares no code with the product path
under nano_vllm_amd/). One function per mechanism, float64 throughout, loops over tokens wherever the design has a mask or a choice.

The design: a decoder whose layers are listed one by one and whose sublayers read the residual stream itself; a sublayer's OUTPUT is
normed, multiplied by a layer scale and added. Attention: the leading entries of q and k turn in pairs (i, i + dims / 2), with
stretched frequencies and a magnitude factor; then q and k are divided by their root mean square per head; sliding window; a learned
sink; from the second value-mixing layer on a layer's values are blended with those of the first one. Feed-forward: a gated unit, or
gated experts chosen by biased logits (weights: softmax over the chosen ones) beside a shared one. The embedding table is the output
matrix.
"""
from __future__ import annotations

import math

import numpy as np


def f64(t) -> np.ndarray:
    import torch
    if isinstance(t, torch.Tensor):
        return t.to(torch.float64).numpy() if t.is_floating_point() else t.numpy().astype(np.int64)
    return np.asarray(t)


def unit_rms(x: np.ndarray, eps: float) -> np.ndarray:
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def silu(z: np.ndarray) -> np.ndarray:
    return z / (1.0 + np.exp(-z))


def branch(x: np.ndarray, y: np.ndarray, w: np.ndarray, scale: np.ndarray, eps: float) -> np.ndarray:
    """The stream after a sublayer whose output is y."""
    return x + unit_rms(y, eps) * w * scale


def frequencies(rot: dict) -> tuple[np.ndarray, float]:
    """(radians per position of every pair, factor on the rotated entries)."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=np.float64)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    factor, orig = float(sc["factor"]), float(sc["original"])
    turns_at = lambda turns: dims * math.log(orig / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(turns_at(float(sc["fast"]))), 0)
    hi = min(math.ceil(turns_at(float(sc["slow"]))), dims - 1)
    for i in range(dims // 2):
        ramp = min(1.0, max(0.0, (i - lo) / max(hi - lo, 0.001)))
        f[i] = f[i] / factor * ramp + f[i] * (1.0 - ramp)
    return f, 0.1 * math.log(factor) + 1.0


def rotate_halves(x: np.ndarray, freq: np.ndarray, mag: float) -> np.ndarray:
    """x [T, heads, d], row t at position t: entries i and i + len(freq) turn by t * freq[i] and grow by mag; the rest pass."""
    out = x.copy()
    half = len(freq)
    pos = np.arange(x.shape[0], dtype=np.float64)
    for i, fi in enumerate(freq):
        c, s = mag * np.cos(pos * fi)[:, None], mag * np.sin(pos * fi)[:, None]
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def mixed_values(v: np.ndarray, first: np.ndarray, lam: float) -> np.ndarray:
    return (1.0 - lam) * v + lam * first


def sink_attention(q: np.ndarray, k: np.ndarray, v: np.ndarray, scale: float, sink: np.ndarray, size: int) -> np.ndarray:
    """q [T, H, d], k [T, G, d], v [T, G, dv]. Row t sees itself and the size - 1 rows before it (size 0: all rows before it); the
    denominator of head a also holds exp(sink[a])."""
    T, H, _ = q.shape
    G, dv = v.shape[1], v.shape[2]
    out = np.zeros((T, H, dv))
    for t in range(T):
        lo = max(0, t - size + 1) if size else 0
        for a in range(H):
            g = a // (H // G)
            s = (k[lo:t + 1, g] @ q[t, a]) * scale
            m = max(s.max(), sink[a])
            e = np.exp(s - m)
            out[t, a] = (e @ v[lo:t + 1, g]) / (e.sum() + math.exp(sink[a] - m))
    return out


def attention(h: np.ndarray, w: dict, m: dict, eps: float, first: np.ndarray | None):
    """(output, this layer's own values before any mixing [T, G, dv]); `first`: the values to mix in, or None."""
    T = h.shape[0]
    H = int(m["heads"])
    G, d = int(m.get("kv_heads", H)), int(m["dim"])
    dv = int(m.get("vdim", d))
    q, k, v = (h @ w["q"].T).reshape(T, H, d), (h @ w["k"].T).reshape(T, G, d), (h @ w["v"].T).reshape(T, G, dv)
    if m.get("rot"):
        freq, mag = frequencies(m["rot"])
        q, k = rotate_halves(q, freq, mag), rotate_halves(k, freq, mag)
    q, k = unit_rms(q, eps), unit_rms(k, eps)
    mixed = v if first is None else mixed_values(v, first, float(w["vmix"]))
    o = sink_attention(q, k, mixed, float(m["scale"]), w["sink"], int((m.get("mask") or {}).get("size", 0)))
    return o.reshape(T, -1) @ w["o"].T, v


def gated_unit(h: np.ndarray, w: dict) -> np.ndarray:
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def _sub(tensors: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def choose(z: np.ndarray, top: int) -> tuple[np.ndarray, np.ndarray]:
    """(experts, weights) of one token's logits."""
    ids = np.argsort(-z, kind="stable")[:top]
    e = np.exp(z[ids] - z[ids].max())
    return ids, e / e.sum()


def experts(h: np.ndarray, w: dict, mlp: dict) -> np.ndarray:
    out = np.zeros_like(h)
    units = [_sub(w, f"e{i}.") for i in range(int(mlp["router"]["experts"]))]
    z = h @ w["router"].T + w["router.b"]
    for t in range(h.shape[0]):
        for i, p in zip(*choose(z[t], int(mlp["router"]["top"]))):
            out[t] += p * gated_unit(h[t:t + 1], units[int(i)])[0]
    if mlp.get("shared"):
        out = out + gated_unit(h, _sub(w, "shared."))
    return out


def forward(raw: dict, tensors: dict, tokens, trace: list | None = None) -> np.ndarray:
    """Logits [T, vocab] of one sequence; `trace` receives the residual rows after every layer."""
    eps = float(raw["norm"]["eps"])
    x = tensors["embed"][np.asarray(tokens)]
    first = None
    for i, layer in enumerate(raw["layers"]):
        assert layer["type"] == "attention"
        w, m, mlp = _sub(tensors, f"l{i}."), layer["mixer"], layer.get("mlp")
        y, v = attention(x, _sub(w, "mix."), m, eps, first if m.get("v_mix") else None)
        if m.get("v_mix") and first is None:
            first = v
        x = branch(x, y, w["norm1"], w["ls1"], eps)
        if mlp is not None:
            wm = _sub(w, "mlp.")
            x = branch(x, experts(x, wm, mlp) if mlp["kind"] == "moe" else gated_unit(x, wm), w["norm2"], w["ls2"], eps)
        if trace is not None:
            trace.append(x.copy())
    return unit_rms(x, eps) * tensors["final.norm"] @ tensors["embed"].T


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
