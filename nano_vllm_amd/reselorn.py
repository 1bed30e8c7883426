"""Reselorn: a decoder-only family whose layers are listed one by one in config.json, with the norm on every sublayer's OUTPUT and a
layer scale. With n(v) = v / sqrt(mean(v^2) + eps) * w, on a 32-bit residual stream:

    x = embed[token]
    x += ls1 * n1(mixer(x));  x += ls2 * n2(ff(x))            (the sublayers read x itself)
    logits = embed n(x)                                       (the embedding table is the output matrix)

Mixer: `attention` (mixers.AttentionMixer: rotation of the leading entries in pairs (i, i + dims / 2) with YaRN-scaled frequencies, heads
normed without weights after the rotation, a sliding window, a learned sink; from the second layer with `v_mix` on, values blended
with those of the first one). Feed-forward: `dense` (SiLU-gated), `moe` (SiLU-gated experts chosen by biased logits, weights a softmax
over the chosen ones, plus a shared expert), or none.

Per-step dataflow on the MI355X (bf16 serving; with dtype float32 every tensor below is 32-bit):

    embed kernel -> x (fp32) and its bf16 copy
    attention:    [q|k|v] GEMM -> store kernel (rotation, norms, scale, value blend, paged K/V) -> attention (window, sink) -> out GEMM
    branch kernel: x += ls1 * n1(mixer), bf16 copy of x
    dense ff:     [gate|up] GEMM -> SiLU GLU kernel -> down GEMM -> branch kernel
    moe ff:       router GEMM (fp32, from x) -> route -> plan -> grouped [gate|up] product (SiLU GLU fused) -> grouped down product; shared
                  expert -> branch kernel, which sums the token's experts and the shared one on the way

Sizes, the layer order and free constants come from config.json; the rule of the YaRN magnitude factor is fixed by the design.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F
from torch import nn

from . import ops_seq
from .attn_meta import get_context
from .mixers import AttentionMixer, BranchNorm, RoutedExperts, SiluGLU, _copy_into, _param, rotary_frequencies


class ReselornConfig:
    """config.json of the family (plus the names of the checkpoint's tensors), with the few attribute names the engine reads from any
    configuration."""

    def __init__(self, raw: dict, tensors=()):
        self.raw, self.tensors = raw, frozenset(tensors)
        self.architecture = raw["architecture"]
        self.vocab_size = int(raw["vocab"])
        self.hidden_size = int(raw["width"])
        self.layers = list(raw["layers"])
        self.num_hidden_layers = len(self.layers)
        self.eps = float(raw["norm"]["eps"])
        self.max_position_embeddings = 1 << 24          # positions are exact integers in a 32-bit float up to here
        self.eos_token_id = raw.get("eos_token_id", -1)
        first = None                                    # (layer, its value heads) of the first value-mixing layer
        for i, layer in enumerate(self.layers):
            if layer["type"] != "attention":
                raise ValueError(f"layer {i}: unknown mixer type {layer['type']!r}")
            mlp = layer.get("mlp")
            if mlp is not None and mlp.get("kind") not in ("dense", "moe"):
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
            heads, kv_heads, _, vdim = head_sizes(layer["mixer"])
            if heads % kv_heads:
                raise ValueError(f"layer {i}: {heads} query heads do not share {kv_heads} key/value heads evenly")
            if layer["mixer"].get("v_mix"):
                first = first or (i, (kv_heads, vdim))
                if first[1] != (kv_heads, vdim):
                    raise ValueError(f"layer {i}: values of {kv_heads} x {vdim} cannot be mixed with those of layer {first[0]}, {first[1][0]} x {first[1][1]}")


def head_sizes(m: dict) -> tuple[int, int, int, int]:
    """(query heads, key/value heads, query/key size, value size) of a mixer."""
    heads, dim = int(m["heads"]), int(m["dim"])
    return heads, int(m.get("kv_heads", heads)), dim, int(m.get("vdim", dim))


def _mixer(width: int, m: dict, eps: float, block_size: int) -> AttentionMixer:
    rot, mask = m.get("rot"), m.get("mask") or {}
    dims = int(rot["dims"]) if rot else 0
    freqs, mag = rotary_frequencies(dims, float(rot["base"]), rot.get("scaling")) if dims else (None, 1.0)
    return AttentionMixer(width, *head_sizes(m), float(m["scale"]), eps, block_size, window=int(mask.get("size") or 0), rot_dims=dims, rot_freqs=freqs,
                          bias=False, sink="learned", rot_halves=True, rot_mag=mag, qk_unit=True, v_mix=bool(m.get("v_mix")))


def _feed_forward(width: int, mlp: dict | None):
    if mlp is None:
        return None
    if mlp["kind"] == "dense":
        return SiluGLU(width, int(mlp["ff"]))
    r, shared = mlp["router"], mlp.get("shared")
    return RoutedExperts(width, int(r["experts"]), int(mlp["expert"]["ff"]), int(r["top"]), shared_ff=int(shared["ff"]) if shared else 0,
                         shared_gate=False, corrected=False, router_bias=True)


class ReselornLayer(nn.Module):

    def __init__(self, width: int, spec: dict, eps: float, block_size: int):
        super().__init__()
        self.mixer = _mixer(width, spec["mixer"], eps, block_size)
        self.mlp = _feed_forward(width, spec.get("mlp"))
        self.routed = isinstance(self.mlp, RoutedExperts)
        self.norm1 = BranchNorm(width, eps)
        self.norm2 = BranchNorm(width, eps) if self.mlp is not None else None

    def named_loaders(self) -> dict:
        out = {"mix." + k: v for k, v in self.mixer.named_loaders().items()}
        out.update({"norm1": _copy_into(self.norm1.w), "ls1": _copy_into(self.norm1.scale)})
        if self.mlp is not None:
            out.update({"mlp." + k: v for k, v in self.mlp.named_loaders().items()})
            out.update({"norm2": _copy_into(self.norm2.w), "ls2": _copy_into(self.norm2.scale)})
        return out


class ReselornForCausalLM(nn.Module):
    stateful = True

    def __init__(self, config: ReselornConfig, dtype=None, block_size: int | None = None):
        super().__init__()
        self.config = config
        self.dtype = dtype or torch.get_default_dtype()
        self.block_size = block_size or getattr(config, "kvcache_block_size", 256)
        self.embed = _param(config.vocab_size, config.hidden_size)
        self.layers = nn.ModuleList(ReselornLayer(config.hidden_size, spec, config.eps, self.block_size) for spec in config.layers)
        self.final_norm = _param(config.hidden_size)
        self.geo = dict(vocab=config.vocab_size, hidden=config.hidden_size, layers=len(config.layers), tie=True)

    def named_loaders(self) -> dict:
        out = {"embed": _copy_into(self.embed), "final.norm": _copy_into(self.final_norm)}
        for i, layer in enumerate(self.layers):
            out.update({f"l{i}.{k}": v for k, v in layer.named_loaders().items()})
            # tensors of what a layer leaves out (no feed-forward, no value mixing) may be in a checkpoint; nothing reads them
            for name in (f"l{i}.norm2", f"l{i}.ls2", f"l{i}.mix.vmix"):
                if name not in out and name in self.config.tensors:
                    out[name] = lambda t: None
        return out

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        """Returns the 32-bit residual stream after the last layer, [n, width]."""
        n, width = input_ids.numel(), self.config.hidden_size
        x = torch.empty(n, width, dtype=torch.float32, device=input_ids.device)
        copy = None if self.dtype == torch.float32 else torch.empty(n, width, dtype=self.dtype, device=x.device)
        xh = x if copy is None else copy                    # what the products read: x itself, or its rounded copy
        ops_seq.embed_sinusoid(self.embed, input_ids, positions, 1.0, 0.0, x, copy)
        trace = getattr(self, "layer_trace", None)          # tests: the residual stream after every layer
        values: list = []                                   # the first value-mixing layer leaves its values here
        for layer in self.layers:
            y = layer.mixer(xh, positions, values if layer.mixer.attn.vmix is not None else None)
            layer.norm1(x, y, copy)
            if layer.mlp is not None:
                y = layer.mlp.parts(xh, wide=x) if layer.routed else layer.mlp(xh)
                layer.norm2(x, y, copy)
            if trace is not None:
                trace.append(x.clone())
        return x

    def compute_logits(self, x: torch.Tensor, rows: torch.Tensor | None = None, nrows: int | None = None) -> torch.Tensor:
        """Logits of the residual rows `rows` (int32 device indices; default: each portion's last token)."""
        if rows is None:
            ctx = get_context()
            nrows = ctx.portions.nseq
            rows = (ctx.portions.cu_q[1:nrows + 1] - 1).to(torch.int32)
        if nrows == 0:
            return torch.empty(0, self.config.vocab_size, dtype=self.dtype, device=x.device)
        normed = torch.empty(nrows, x.shape[1], dtype=self.dtype, device=x.device)
        ops_seq.offset_norm_rows(x, rows, nrows, self.final_norm, self.config.eps, normed, w_off=0.0)
        return F.linear(normed, self.embed)


# ---- synthetic checkpoints (tests, benchmarks, dummy weights) -----------------------------------------------------------
def tensor_shapes(raw: dict) -> dict[str, tuple]:
    """Checkpoint tensor names -> shapes of a configuration (the parsed config.json)."""
    W, V = raw["width"], raw["vocab"]
    out = {"embed": (V, W), "final.norm": (W,)}
    for i, layer in enumerate(raw["layers"]):
        p, mlp = f"l{i}.", layer.get("mlp")
        H, G, d, dv = head_sizes(layer["mixer"])
        out.update({p + "norm1": (W,), p + "ls1": (W,), p + "mix.q": (H * d, W), p + "mix.k": (G * d, W), p + "mix.v": (G * dv, W),
                    p + "mix.sink": (H,), p + "mix.o": (W, H * dv)})
        if layer["mixer"].get("v_mix"):
            out[p + "mix.vmix"] = ()
        if mlp is None:
            continue
        out.update({p + "norm2": (W,), p + "ls2": (W,)})

        def unit(name: str, ff: int) -> None:
            out.update({f"{p}mlp.{name}gate": (ff, W), f"{p}mlp.{name}up": (ff, W), f"{p}mlp.{name}down": (W, ff)})
        if mlp["kind"] == "dense":
            unit("", mlp["ff"])
            continue
        E = mlp["router"]["experts"]
        for e in range(E):
            unit(f"e{e}.", mlp["expert"]["ff"])
        out.update({p + "mlp.router": (E, W), p + "mlp.router.b": (E,)})
        if mlp.get("shared"):
            unit("shared.", mlp["shared"]["ff"])
    return out


def random_tensors(raw: dict, seed: int = 0) -> dict[str, torch.Tensor]:
    """Seeded random bf16 weights in ranges that keep every mechanism alive: matrices scaled by their fan-in, norm weights around
    one, layer scales around a half, sinks and router biases of order one, mixing factors between 0 and 1."""
    gen = torch.Generator(device="cpu").manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(raw).items():
        leaf = name.split(".")[-1]
        r = torch.randn(shape, generator=gen, dtype=torch.float32, device="cpu")
        if leaf in ("norm", "norm1", "norm2"):
            t = 1.0 + 0.1 * r
        elif leaf in ("ls1", "ls2"):
            t = 0.5 + 0.1 * r
        elif leaf == "vmix":
            t = torch.sigmoid(r)
        elif leaf in ("sink", "b") or name == "embed":
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


ReselornForCausalLM.init_random = _init_random
