"""Ligidra: a decoder-only family whose layers are listed one by one in config.json, on a 32-bit residual stream with three
branches per layer. With n(v) = v / sqrt(mean(v^2) + eps) * w:

    x = n(embed[token])
    h = n1(x);  x += mixer(h + (h of the previous token - h) * shift)
    x += ff(n2(x))
    x += n_side(W_proj (gelu(W_gate x) * side[token, layer's part]))
    logits = embed n(x)                                          (the embedding table is the output matrix)

Mixers: `attention` (mixers.AttentionMixer: q / k norms over the whole projection, band-wise scaled rotation, capped scores, a
learned sink, a sliding window with pooled blocks behind it; with `kv_from: j` layer j's cached keys and values), `delta` (one decay
per head, SiLU gate) and `channel_delta` (a decay per head and key channel and a sigmoid gate, both low-rank), both
mixers.DeltaMixer. Feed-forward: `moe` (softmax-routed experts with the scores as weights, plus a shared expert), or none.

Per-step dataflow on the MI355X (bf16 serving; with dtype float32 every tensor below is 32-bit):

    embed + norm kernel -> x (fp32)
    shift-norm kernel:  x' = x + n_side(previous layer's side branch); h = n1(x') blended with the previous token's  — one launch
    attention:          [q|k|v] GEMM -> row norms + rotation + paged K/V store (+ block means) -> attention (q norm, rotation, cap,
                        sink, window and pooled blocks fused) -> out GEMM
    delta:              [q|k|v|g|a|b] GEMM -> causal convolution + SiLU -> delta scan (fp32 state) -> per-head norm + gate -> out GEMM
    norm kernel:        x' += mixer; n2(x')
    moe:                router GEMM (fp32) -> route -> plan -> grouped [gate|up] product (SiLU GLU fused) -> grouped down product ->
                        combine kernel (weights, shared expert, the residual add, x' in bf16)
    side:               gate GEMM -> gated lookup kernel -> projection GEMM (its norm and add: the next shift-norm kernel)

Sizes, the layer order and free constants come from config.json, the ranks of the low-rank projections from the tensors'
shapes; the 1e-6 of the unit vectors and the GELU's constants are fixed by the design.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F
from torch import nn

from . import ops_seq
from .attn_meta import get_context
from .mixers import (AttentionMixer, DeltaMixer, RoutedExperts, TokenShiftNorm, TokenSide, _copy_into, _param,
                     banded_rotary_frequencies)


class LigidraConfig:
    """config.json of the family (plus the shapes of the checkpoint's tensors, for the ranks that only they tell), with the few
    attribute names the engine reads from any configuration. Without a checkpoint, ranks are the mixer's
    `decay_rank` / `gate_rank`, or its `dim`."""

    def __init__(self, raw: dict, shapes: dict | None = None):
        self.raw, self.shapes = raw, shapes or {}
        self.architecture = raw["architecture"]
        self.vocab_size = int(raw["vocab"])
        self.hidden_size = int(raw["width"])
        self.layers = list(raw["layers"])
        self.num_hidden_layers = len(self.layers)
        self.eps = float(raw["norm"]["eps"])
        side = raw.get("token_side")
        self.side_dim = int(side["dim"]) if side else 0
        self.max_position_embeddings = 1 << 24          # positions are exact integers in a 32-bit float up to here
        self.eos_token_id = raw.get("eos_token_id", -1)
        for i, layer in enumerate(self.layers):
            if layer["type"] not in ("attention", "delta", "channel_delta"):
                raise ValueError(f"layer {i}: unknown mixer type {layer['type']!r}")
            mlp = layer.get("mlp")
            if mlp is not None and mlp.get("kind") != "moe":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
            src = layer["mixer"].get("kv_from")
            if src is not None:
                src = int(src)
                if not (0 <= src < i) or self.layers[src]["type"] != "attention" or self.layers[src]["mixer"].get("kv_from") is not None:
                    raise ValueError(f"layer {i}: kv_from {src} must name an earlier attention layer with projections of its own")

    def ranks(self, i: int) -> tuple[int, int]:
        """Ranks of the decay and the gate projection of a channel_delta layer."""
        m = self.layers[i]["mixer"]
        return tuple(int(self.shapes.get(f"l{i}.mix.{t}", (m.get(key, m["dim"]),))[0]) for t, key in (("a1", "decay_rank"), ("g1", "gate_rank")))


def _mixer(config: LigidraConfig, i: int, block_size: int, sources: list):
    width, eps = config.hidden_size, config.eps
    kind, m = config.layers[i]["type"], config.layers[i]["mixer"]
    heads, dim = int(m["heads"]), int(m["dim"])
    kv_heads, vdim = int(m.get("kv_heads", heads)), int(m.get("vdim", dim))
    if kind == "attention":
        rot, mask = m.get("rot"), m.get("mask") or {}
        dims = int(rot["dims"]) if rot else 0
        return AttentionMixer(width, heads, kv_heads, dim, vdim, m["scale"], eps, block_size, window=int(mask.get("size", 0)), rot_dims=dims,
                              qk_norm=True, bias=False, source=sources[int(m["kv_from"])] if m.get("kv_from") is not None else None,
                              rot_freqs=banded_rotary_frequencies(dims, float(rot["base"]), rot.get("scaling")) if rot else None,
                              sink="learned", norm_rows=True, softcap=float(m.get("softcap") or 0.0), pool=int(mask.get("pool") or 0))
    decay_rank, gate_rank = config.ranks(i) if kind == "channel_delta" else (0, 0)
    return DeltaMixer(width, heads, kv_heads, dim, vdim, int(m.get("conv", 1)), eps, decay_rank, gate_rank)


class LigidraLayer(nn.Module):

    def __init__(self, config: LigidraConfig, i: int, block_size: int, sources: list):
        super().__init__()
        width, mlp = config.hidden_size, config.layers[i].get("mlp")
        self.mixer = _mixer(config, i, block_size, sources)
        self.norm1 = TokenShiftNorm(width, config.eps)
        self.mlp = self.norm2 = self.side = None
        if mlp is not None:
            r, shared = mlp["router"], mlp.get("shared")
            self.mlp = RoutedExperts(width, int(r["experts"]), int(mlp["expert"]["ff"]), int(r["top"]), shared_ff=int(shared["ff"]) if shared else 0,
                                     renorm=False, shared_gate=False, corrected=False)
            self.norm2 = _param(width)
        if config.side_dim:
            self.side = TokenSide(width, config.side_dim, i * config.side_dim)

    def named_loaders(self) -> dict:
        out = {"mix." + k: v for k, v in self.mixer.named_loaders().items()}
        out.update({"norm1": _copy_into(self.norm1.w), "shift": _copy_into(self.norm1.shift)})
        if self.mlp is not None:
            out.update({"mlp." + k: v for k, v in self.mlp.named_loaders().items()})
            out["norm2"] = _copy_into(self.norm2)
        if self.side is not None:
            out.update({"side." + k: v for k, v in self.side.named_loaders().items()})
        return out


class LigidraForCausalLM(nn.Module):
    stateful = True

    def __init__(self, config: LigidraConfig, dtype=None, block_size: int | None = None):
        super().__init__()
        self.config = config
        self.dtype = dtype or torch.get_default_dtype()
        self.block_size = block_size or getattr(config, "kvcache_block_size", 256)
        width = config.hidden_size
        self.embed, self.embed_norm, self.final_norm = _param(config.vocab_size, width), _param(width), _param(width)
        self.side_embed = _param(config.vocab_size, len(config.layers) * config.side_dim) if config.side_dim else None
        self.layers = nn.ModuleList()
        for i in range(len(config.layers)):
            self.layers.append(LigidraLayer(config, i, self.block_size, [layer.mixer for layer in self.layers]))
        self.geo = dict(vocab=config.vocab_size, hidden=width, layers=len(config.layers), tie=True)

    def named_loaders(self) -> dict:
        out = {"embed": _copy_into(self.embed), "embed.norm": _copy_into(self.embed_norm), "final.norm": _copy_into(self.final_norm)}
        if self.side_embed is not None:
            out["side.embed"] = _copy_into(self.side_embed)
        for i, layer in enumerate(self.layers):
            out.update({f"l{i}.{k}": v for k, v in layer.named_loaders().items()})
        return out

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> tuple:
        """Returns what compute_logits takes: the 32-bit residual stream [n, width] before the last layer's last branch, that branch, and
        the weight of the norm on it (None: it is added as it is). A layer's last branch is always added by the kernel that norms the
        stream next; the last one only for the rows whose logits are asked for."""
        n, cfg = input_ids.numel(), self.config
        x = torch.empty(n, cfg.hidden_size, dtype=torch.float32, device=input_ids.device)
        ops_seq.embed_norm(self.embed, input_ids, self.embed_norm, cfg.eps, x)
        trace = getattr(self, "layer_trace", None)          # tests: the residual stream after every layer
        wide = self.dtype == torch.float32

        def add(x, a, wa):
            if wa is not None:
                ops_seq.sandwich_norm(x, a, wa, None, cfg.eps, None, w_off=0.0)
            else:
                ops_seq.add_group_norm(x, None, 1, cfg.eps, None, a)
            return x

        pending = (None, None)
        for layer in self.layers:
            x, h = layer.norm1(x, *pending, self.dtype)
            y = layer.mixer(h, positions)
            pending, xh = (None, None), None
            if layer.mlp is not None:
                h = torch.empty(n, cfg.hidden_size, dtype=self.dtype, device=x.device)
                ops_seq.add_group_norm(x, layer.norm2, 1, cfg.eps, h, y)
                xh = layer.mlp(h, res=x)
            elif layer.side is not None:
                xh = x if wide else torch.empty(n, cfg.hidden_size, dtype=self.dtype, device=x.device)
                ops_seq.add_group_norm(x, None, 1, cfg.eps, None if wide else xh, y)
            else:
                pending = (y, None)
            if layer.side is not None:
                pending = (layer.side(xh, self.side_embed, input_ids), layer.side.norm)
            if trace is not None:
                if pending[0] is not None:
                    x, pending = add(x, *pending), (None, None)
                trace.append(x.clone())
        if pending[0] is not None and pending[1] is None:
            x, pending = add(x, *pending), (None, None)
        return x, *pending

    def compute_logits(self, hidden: tuple, rows: torch.Tensor | None = None, nrows: int | None = None) -> torch.Tensor:
        """Logits of the rows `rows` (int32 device indices; default: each portion's last token) of what forward() returned."""
        x, branch, wa = hidden
        if rows is None:
            ctx = get_context()
            nrows = ctx.portions.nseq
            rows = (ctx.portions.cu_q[1:nrows + 1] - 1).to(torch.int32)
        if nrows == 0:
            return torch.empty(0, self.config.vocab_size, dtype=self.dtype, device=x.device)
        normed = torch.empty(nrows, x.shape[1], dtype=self.dtype, device=x.device)
        ops_seq.offset_norm_rows(x, rows, nrows, self.final_norm, self.config.eps, normed, w_off=0.0, a=branch, wa=wa)
        return F.linear(normed, self.embed)


# ---- synthetic checkpoints (tests, benchmarks, dummy weights) -----------------------------------------------------------
def tensor_shapes(raw: dict) -> dict[str, tuple]:
    """Checkpoint tensor names -> shapes of a configuration (the parsed config.json). Low ranks: the mixer's
    `decay_rank` / `gate_rank`, or its `dim`."""
    W, V = raw["width"], raw["vocab"]
    out = {"embed": (V, W), "embed.norm": (W,), "final.norm": (W,)}
    side = raw.get("token_side")
    if side:
        out["side.embed"] = (V, len(raw["layers"]) * side["dim"])
    for i, layer in enumerate(raw["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        H, d = m["heads"], m["dim"]
        G, dv = m.get("kv_heads", H), m.get("vdim", d)
        out.update({p + "norm1": (W,), p + "shift": (W,), p + "mix.q": (H * d if layer["type"] == "attention" else G * d, W), p + "mix.o": (W, H * dv)})
        if layer["type"] == "attention":
            out.update({p + "mix.q.norm": (H * d,), p + "mix.sink": (H,)})
            if m.get("kv_from") is None:
                out.update({p + "mix.k": (G * d, W), p + "mix.v": (G * dv, W), p + "mix.k.norm": (G * d,)})
        else:
            taps, channelwise = m.get("conv", 1), layer["type"] == "channel_delta"
            out.update({p + "mix.k": (G * d, W), p + "mix.v": (H * dv, W), p + "mix.q.conv": (G * d, taps), p + "mix.k.conv": (G * d, taps),
                        p + "mix.v.conv": (H * dv, taps), p + "mix.b": (H, W), p + "mix.A_log": (H,), p + "mix.norm": (dv,),
                        p + "mix.dt_bias": (H * d if channelwise else H,)})
            if channelwise:
                ar, gr = m.get("decay_rank", d), m.get("gate_rank", d)
                out.update({p + "mix.a1": (ar, W), p + "mix.a2": (H * d, ar), p + "mix.g1": (gr, W), p + "mix.g2": (H * dv, gr)})
            else:
                out.update({p + "mix.a": (H, W), p + "mix.g": (H * dv, W)})
        mlp = layer.get("mlp")
        if mlp is not None:
            out[p + "norm2"] = (W,)
            ff = mlp["expert"]["ff"]
            for e in range(mlp["router"]["experts"]):
                out.update({p + f"mlp.e{e}.gate": (ff, W), p + f"mlp.e{e}.up": (ff, W), p + f"mlp.e{e}.down": (W, ff)})
            out[p + "mlp.router"] = (mlp["router"]["experts"], W)
            if mlp.get("shared"):
                sf = mlp["shared"]["ff"]
                out.update({p + "mlp.shared.gate": (sf, W), p + "mlp.shared.up": (sf, W), p + "mlp.shared.down": (W, sf)})
        if side:
            out.update({p + "side.gate": (side["dim"], W), p + "side.proj": (W, side["dim"]), p + "side.norm": (W,)})
    return out


def random_tensors(raw: dict, seed: int = 0) -> dict[str, torch.Tensor]:
    """Seeded random bf16 weights in ranges that keep every mechanism alive: matrices scaled by their fan-in, norm weights around
    one, shifts between 0 and 1, sinks of order one, decays spread between fast and slow."""
    gen = torch.Generator(device="cpu").manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(raw).items():
        leaf = name.split(".")[-1]
        r = torch.randn(shape, generator=gen, dtype=torch.float32, device="cpu")
        if leaf in ("norm", "norm1", "norm2"):
            t = 1.0 + 0.1 * r
        elif leaf == "shift":
            t = torch.sigmoid(r)
        elif leaf == "sink":
            t = r
        elif leaf == "A_log":
            t = -1.0 + 0.7 * r
        elif leaf == "dt_bias":
            t = -2.0 + r
        elif leaf == "conv":
            t = r / (shape[-1] ** 0.5)
        elif name in ("embed", "side.embed"):
            t = r
        else:
            t = r / (shape[-1] ** 0.5)
        out[name] = t.to(torch.bfloat16)
    return out


def write_synthetic_checkpoint(path: str, raw: dict, seed: int = 0, tensors: dict | None = None) -> str:
    """config.json + model.safetensors of a random model of the family (no tokenizer: requests are token ids)."""
    import json
    import os
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as fh:
        json.dump(raw, fh, indent=1)
    tensors = tensors if tensors is not None else random_tensors(raw, seed)
    save_file({k: v.contiguous() for k, v in tensors.items()}, os.path.join(path, "model.safetensors"))
    return path


def _init_random(self, seed: int = 0) -> None:
    loaders = self.named_loaders()
    dev = self.embed.device
    for name, t in random_tensors(self.config.raw, seed).items():
        loaders[name](t.to(dev))


LigidraForCausalLM.init_random = _init_random
