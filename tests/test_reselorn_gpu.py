"""Reselorn on the GPU against the plain float64 restatement (oracle/reselorn.py): every mechanism alone at the kernel or layer
boundary, then the engine — whole prompts, portions down to two tokens, token-by-token decoding, unequal batches, reused pages and
slots, window edges, far keys, sinks, the first tokens, long decoding, greedy generation through LLM.generate(). Configurations and
weights are made here; float32 serving is compared tightly, bfloat16 serving within rounding (where a choice of experts could
depend on rounding, every expert is chosen)."""
import json
import math
import os
import subprocess
import sys
import tempfile

import numpy as np
import pytest
import torch

pytestmark = pytest.mark.gpu

from oracle import reselorn as plain  # noqa: E402

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
EPS = 1e-5
F32, BF16 = torch.float32, torch.bfloat16
BOTH = [(F32, 3e-6), (BF16, 2.0 ** -8)]
LAYER_BOTH = [(F32, 3e-5), (BF16, 3e-2)]


def dev(t, dtype=None):
    return t.to("cuda", dtype=dtype or t.dtype).contiguous()


def bf(t):
    return t.to(torch.bfloat16)


def normal(seed):
    g = torch.Generator().manual_seed(seed)
    return lambda *s: torch.randn(*s, generator=g)


def close(got, want, tol, what=""):
    got = got.double().cpu().numpy() if hasattr(got, "cpu") else np.asarray(got, dtype=np.float64)
    want = want.double().cpu().numpy() if hasattr(want, "cpu") else np.asarray(want, dtype=np.float64)
    err = np.abs(got - want).max() / max(np.abs(want).max(), 1e-9)
    assert err <= tol, f"{what}: relative error {err:.3e} > {tol:.1e}"


def portions(lens, ctx0, slots):
    from nano_vllm_amd.ops_seq import Portions
    cu = np.concatenate([[0], np.cumsum(lens)]).astype(np.int32)
    tseq = np.repeat(np.arange(len(lens)), lens).astype(np.int32)
    i32 = lambda a: torch.tensor(np.asarray(a, dtype=np.int32), device="cuda")
    return Portions(i32(cu), i32(ctx0), i32(slots), i32(tseq), len(lens), int(cu[-1]), max(lens))


# ---------------------------------------------------------------------------------------------- rotation, norms, blend, store
def turned(x, pos, freq, mag, halves):
    """x [n, heads, d] at the positions pos, in either pairing (the oracle's rotation is at positions 0, 1, .. and by halves only). Angles
    are products in 32-bit, as the design has them."""
    out, half = x.copy(), len(freq)
    for i, f in enumerate(freq):
        a, b = (i, i + half) if halves else (2 * i, 2 * i + 1)
        angle = (pos.astype(np.float32) * np.float32(f)).astype(np.float64)[:, None]
        c, s = mag * np.cos(angle), mag * np.sin(angle)
        out[..., a], out[..., b] = x[..., a] * c - x[..., b] * s, x[..., b] * c + x[..., a] * s
    return out


@pytest.mark.parametrize("dtype,tol", [(F32, 2e-6), (BF16, 2.0 ** -7)])
@pytest.mark.parametrize("H,G,d,dv,rot,halves,unit,blend,block,n", [
    (4, 2, 24, 40, 16, True, True, True, 16, 5),           # eight entries per lane, a head that is no power of two
    (3, 1, 64, 64, 64, True, True, False, 32, 600),        # everything turns; tiles of 8 tokens
    (6, 3, 128, 16, 32, True, True, True, 64, 2100),       # tiles of 32 tokens
    (2, 2, 40, 72, 20, True, True, True, 16, 2053),        # pairs that do not fall into whole units of eight
    (5, 5, 9, 7, 6, True, True, True, 16, 33),             # nothing divisible by anything
    (2, 1, 21, 130, 0, True, True, False, 48, 700),        # no rotation
    (2, 2, 64, 24, 24, False, False, True, 16, 530),       # neighbours as pairs, no norm
    (1, 1, 8, 8, 8, False, True, False, 16, 40),
    (2, 1, 264, 200, 144, True, True, True, 16, 601), (1, 1, 512, 8, 512, True, True, False, 16, 30),
    (2, 1, 600, 520, 600, True, True, True, 16, 9),        # long heads
    (20, 10, 96, 32, 80, True, False, True, 16, 71), (1, 1, 256, 256, 256, True, True, True, 64, 2050)])
def test_rotation_norm_scale_blend_and_store(H, G, d, dv, rot, halves, unit, blend, block, n, dtype, tol):
    """Two portions with a cut inside a page between them, pages in scattered order, a few rows that are not stored; what was in the
    cache beside the written places stays."""
    from nano_vllm_amd import ops_seq
    rnd = normal(H * 1000 + d + n)
    qc, kc, vc = H * d, G * d, G * dv
    proj, first = bf(rnd(n, qc + kc + vc)), bf(rnd(n, vc + 8))
    lam, mag, scale = 0.3125, 1.25, 0.37
    cut = n // 3
    pos = torch.cat([torch.arange(3, 3 + cut), torch.arange(1200, 1200 + n - cut)])
    pages = -(-(n + 1300) // block)
    table = torch.randperm(pages, generator=torch.Generator().manual_seed(1))
    places = torch.cat([pos[:cut], pos[cut:] - 1200 + cut + 8])      # the second portion right behind the first, five places further
    slots = (table[places // block] * block + places % block).to(torch.int32)
    slots[[0, n // 2]] = -1
    freq = torch.tensor([100.0 ** (-2.0 * i / rot) * 0.7 for i in range(rot // 2)], dtype=torch.float32)
    p = dev(proj, dtype)
    kcache = torch.full((pages * block, G, d), 5.0, dtype=dtype, device="cuda")
    vcache = torch.full((pages * block, G, dv), 6.0, dtype=dtype, device="cuda")
    r = ops_seq.Rotation(dev(freq), halves, mag) if rot else None
    ops_seq.qkv_store(p[:, :qc], p[:, qc:qc + kc], p[:, qc + kc:], H, G, d, dv, block, dev(slots), kcache, vcache, dev(pos) if rot else None, r, unit, EPS,
                      scale, dev(first, dtype)[:, :vc] if blend else None, torch.tensor(lam, device="cuda") if blend else None)
    f = plain.f64(proj)
    q, k, v = f[:, :qc].reshape(n, H, d), f[:, qc:qc + kc].reshape(n, G, d), f[:, qc + kc:].reshape(n, G, dv)
    fr, ps = plain.f64(freq), plain.f64(pos).astype(np.float64)
    q, k = (turned(t, ps, fr, mag, halves) for t in (q, k))
    if unit:
        q, k = plain.unit_rms(q, EPS), plain.unit_rms(k, EPS)
    if blend:
        v = plain.mixed_values(v, plain.f64(first)[:, :vc].reshape(n, G, dv), lam)
    close(p[:, :qc].float(), (q * scale).reshape(n, -1), tol, "queries")
    assert torch.equal(p[:, qc:].cpu(), proj.to(dtype)[:, qc:]), "keys and values of the projection are only read"
    wk, wv = np.full((pages * block, G, d), 5.0), np.full((pages * block, G, dv), 6.0)
    stored = (slots >= 0).numpy()
    wk[slots.numpy()[stored]], wv[slots.numpy()[stored]] = k[stored], v[stored]
    close(kcache, wk, tol, "keys")
    vt = vcache.view(pages, G, dv, block).permute(0, 3, 1, 2).reshape(pages * block, G, dv)      # values are transposed inside a page
    close(vt, wv, tol, "values")


@pytest.mark.parametrize("scaling", [None, {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}, {"factor": 16.0, "original": 4096, "fast": 32.0, "slow": 1.0},
                                     {"factor": 2.0, "original": 16, "fast": 1.0, "slow": 1.0}])
@pytest.mark.parametrize("dims,base", [(8, 100.0), (56, 10000.0), (2, 50.0)])
def test_stretched_frequencies(dims, base, scaling):
    from nano_vllm_amd.mixers import rotary_frequencies
    freq, mag = rotary_frequencies(dims, base, scaling)
    want, wmag = plain.frequencies({"dims": dims, "base": base, "scaling": scaling})
    close(torch.tensor(freq, dtype=torch.float64), want, 1e-14)
    assert mag == pytest.approx(wmag, abs=1e-15) and (scaling is not None or mag == 1.0)


# ---------------------------------------------------------------------------------------------- branch, activation, lookup
@pytest.mark.parametrize("dtype,tol", BOTH)
@pytest.mark.parametrize("W", [4, 50, 260, 1028, 4096, 5000, 8192, 9001, 16384])
@pytest.mark.parametrize("kind", ["plain", "no scale", "chosen", "both"])
def test_a_normed_branch_with_a_layer_scale(dtype, tol, W, kind):
    from nano_vllm_amd import ops_seq
    n, top, cap = 7, 3, 32
    rnd = normal(W)
    x, a, rows, w, ls = rnd(n, W), bf(rnd(n, W)), bf(rnd(cap, W)), bf(1 + 0.2 * rnd(W)), bf(0.4 + 0.2 * rnd(W))
    wts = torch.rand(n, top, generator=torch.Generator().manual_seed(3))
    pair = torch.randperm(cap, generator=torch.Generator().manual_seed(4))[:n * top].view(n, top).to(torch.int32)
    pair[2, 1] = -1                                                  # a choice without a row adds nothing
    y = np.zeros((n, W))
    if kind != "chosen":
        y = y + plain.f64(a)
    plan = chosen = None
    if kind in ("chosen", "both"):
        full = np.where((pair >= 0).numpy()[..., None], plain.f64(rows)[pair.clamp(min=0).numpy()], 0.0)
        y = y + (full * plain.f64(wts)[..., None]).sum(1)
        plan = ops_seq.MoePlan()
        plan.pair_row = dev(pair)
        chosen = (dev(rows, dtype), plan, dev(wts))
    scale = plain.f64(ls) if kind != "no scale" else 1.0
    want = plain.branch(plain.f64(x), y, plain.f64(w), scale, EPS)
    gx, out = dev(x), torch.empty(n, W, dtype=dtype, device="cuda")
    ops_seq.branch_norm(gx, dev(a, dtype) if kind != "chosen" else None, dev(w, dtype), dev(ls, dtype) if kind != "no scale" else None, EPS, out, chosen)
    close(gx, want, 3e-6, "stream")                                  # (32-bit in both modes)
    assert torch.equal(out, gx.to(dtype))
    g2 = dev(x)
    ops_seq.branch_norm(g2, dev(a, dtype) if kind != "chosen" else None, dev(w, dtype), dev(ls, dtype) if kind != "no scale" else None, EPS, None, chosen)
    assert torch.equal(g2, gx)


@pytest.mark.parametrize("dtype,tol", [(F32, 2e-6), (BF16, 2.0 ** -7)])
@pytest.mark.parametrize("n,ff,pad", [(5, 24, 0), (130, 64, 16), (3, 7, 1), (1, 1000, 4), (40, 12, 0)])
def test_gated_activation_and_plain_lookup(n, ff, pad, dtype, tol):
    from nano_vllm_amd import ops_seq
    rnd = normal(ff)
    gu = bf(2 * rnd(n, 2 * ff + pad))
    out = torch.empty(n, ff, dtype=dtype, device="cuda")
    ops_seq.glu_act(dev(gu, dtype)[:, :2 * ff], ff, out, kind=0)
    f = plain.f64(gu)
    close(out, plain.silu(f[:, :ff]) * f[:, ff:2 * ff], tol)
    ops_seq.glu_act(dev(gu, dtype)[:, :2 * ff], ff, out, kind=1, limit=1.5, alpha=1.7)
    g, u = np.minimum(f[:, :ff], 1.5), np.clip(f[:, ff:2 * ff], -1.5, 1.5)
    close(out, g / (1 + np.exp(-1.7 * g)) * (u + 1), tol, "clamped")
    ops_seq.glu_act(dev(gu, dtype)[:, :ff], ff, out, kind=2)
    close(out, 0.5 * f[:, :ff] * (1 + np.tanh(math.sqrt(2 / math.pi) * (f[:, :ff] + 0.044715 * f[:, :ff] ** 3))), tol, "ungated")
    table, ids = bf(rnd(11, ff)), torch.randint(0, 11, (n,), generator=torch.Generator().manual_seed(0))
    x, xh = torch.empty(n, ff, device="cuda"), torch.empty(n, ff, dtype=dtype, device="cuda")
    ops_seq.embed_sinusoid(dev(table, dtype), dev(ids), dev(torch.zeros(n, dtype=torch.int64)), 1.0, 0.0, x, xh)
    assert torch.equal(x.cpu(), table.float()[ids]) and torch.equal(xh, x.to(dtype))


# ---------------------------------------------------------------------------------------------- layers in a step's context
def with_context(mix, h, dtype, block, cuts, path="auto", values=None):
    """Run a layer on the rows of h in portions `cuts`, through pages in scattered order that hold something else before; `values`: rows
    of an earlier layer's values to mix in."""
    from nano_vllm_amd import ops_seq
    from nano_vllm_amd.attn_meta import reset_context, set_context
    T = h.shape[0]
    pages = -(-T // block)
    order = torch.randperm(pages + 3, generator=torch.Generator().manual_seed(2))[:pages].to(torch.int32)
    mod = mix.attn
    ks, vs = mod.kv_shapes()
    mod.block_size = block
    mod.k_cache = torch.full(((pages + 3) * block, *ks), 2.0, dtype=dtype, device="cuda")
    mod.v_cache = torch.full(((pages + 3) * block, *vs), -2.0, dtype=dtype, device="cuda")
    ops_seq.load_library().nvs_window_attn_force_scalar({"auto": 0, "scalar": 1, "no_lds": 2, "unpacked": 3}[path])
    outs, at = [], 0
    try:
        with torch.inference_mode():
            for c in cuts:
                pos = torch.arange(at, at + c)
                slots = (order[pos // block].long() * block + pos % block).to(torch.int32)
                set_context(True, slot_mapping=dev(slots), block_tables=dev(order.view(1, -1)), portions=portions([c], [at], [1]))
                vals = [dev(values[at:at + c], dtype)] if values is not None else ([] if mod.vmix is not None else None)
                outs.append(mix(dev(h[at:at + c], dtype), dev(pos), vals).float().cpu())
                if values is None and vals is not None:
                    assert len(vals) == 1 and vals[0].shape == (c, mod.G * mod.dv)      # the first layer leaves its values
                at += c
    finally:
        reset_context()
        ops_seq.load_library().nvs_window_attn_force_scalar(0)
    assert at == T
    return torch.cat(outs)


def build(cls, w, dtype, *args, **kw):
    with torch.inference_mode():
        prev = torch.get_default_dtype()
        torch.set_default_dtype(dtype)
        try:
            mix = cls(*args, **kw).to("cuda")
        finally:
            torch.set_default_dtype(prev)
        loaders = mix.named_loaders()
        assert set(loaders) == set(w), sorted(set(loaders) ^ set(w))
        for k, fn in loaders.items():
            fn(w[k].to("cuda"))
    return mix


ROT = {"dims": 8, "base": 100.0, "scaling": {"factor": 4.0, "fast": 4.0, "slow": 1.0, "original": 64}}


def attention_case(H, G, d, dv, size, rot_dims, T, seed, W=40, sharp=1.5):
    rnd = normal(seed)
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": sharp * d ** -0.5, "v_mix": True}
    if size:
        m["mask"] = {"size": size}
    if rot_dims:
        m["rot"] = dict(ROT, dims=rot_dims)
    w = {"q": rnd(H * d, W) / W ** 0.5, "k": rnd(G * d, W) / W ** 0.5, "v": rnd(G * dv, W) / W ** 0.5, "o": rnd(W, H * dv) / (H * dv) ** 0.5,
         "sink": 1 + rnd(H), "vmix": torch.tensor(0.4)}
    return m, {k: bf(v) for k, v in w.items()}, bf(rnd(T, W))


def build_attention(m, w, dtype, block, W=40):
    from nano_vllm_amd.reselorn import _mixer
    return build(lambda: _mixer(W, m, EPS, block), w, dtype)


def plain_attention(h, w, m, first=None):
    return plain.attention(plain.f64(h), {k: plain.f64(v) for k, v in w.items()}, m, EPS, first)


@pytest.mark.parametrize("dtype,path,tol", [(F32, "auto", 3e-5), (BF16, "auto", 3e-2), (BF16, "scalar", 3e-2), (BF16, "unpacked", 3e-2), (BF16, "no_lds", 3e-2)])
@pytest.mark.parametrize("H,G,d,dv,size,block,rot_dims", [
    (4, 2, 16, 24, 24, 16, 8), (8, 1, 24, 16, 7, 32, 16), (3, 3, 20, 12, 40, 16, 4), (2, 1, 64, 80, 1, 16, 0), (1, 1, 40, 40, 33, 16, 16),
    (6, 2, 136, 72, 16, 64, 48), (2, 2, 16, 200, 500, 48, 16), (20, 2, 8, 8, 50, 64, 8), (4, 4, 96, 32, 2, 16, 96), (6, 3, 32, 8, 0, 16, 32),
    (2, 1, 256, 256, 26, 32, 128), (1, 1, 280, 264, 20, 16, 64)])
def test_windowed_attention_with_a_sink_and_mixed_values(H, G, d, dv, size, block, rot_dims, dtype, path, tol):
    T = 150
    m, w, h = attention_case(H, G, d, dv, size, rot_dims, T, seed=H * 100 + d)
    first = bf(normal(9)(T, G * dv))
    want = plain_attention(h, w, m, plain.f64(first).reshape(T, G, dv))[0]
    for cuts in ([T], [77, 2, 1, 1, 30, 2, 1, 1, 1, 34], [1] * 30 + [2] * 20 + [80]):
        close(with_context(build_attention(m, w, dtype, block), h, dtype, block, cuts, path, first), want, tol, f"cuts {cuts[:3]}")
    if path == "auto":                                               # as the first value-mixing layer, and without value mixing
        own = plain_attention(h, w, m)[0]
        close(with_context(build_attention(m, w, dtype, block), h, dtype, block, [70, 1, 79]), own, tol, "first")
        close(with_context(build_attention(dict(m, v_mix=False), {k: v for k, v in w.items() if k != "vmix"}, dtype, block), h, dtype, block, [T]), own, tol,
              "unmixed")


def marked_case(T, size, key_at, d=16, W=32, H=2):
    """Every query looks along the last entry, which does not turn, and the token `key_at` alone has a key along it and a value that
    stands out: wherever it is seen, the output shows it."""
    rnd = normal(T + key_at)
    m = {"heads": H, "kv_heads": 1, "dim": d, "vdim": d, "scale": 0.75, "mask": {"size": size}, "v_mix": False, "rot": dict(ROT)}
    h = 0.3 * rnd(T, W)
    h[:, :2] = 0.0
    h[:, 0] = 3.0
    h[key_at, 1] = 12.0
    u = torch.zeros(d)
    u[-1] = 1.0
    q, k, v = 0.02 * rnd(H * d, W), 0.3 * rnd(d, W), 0.3 * rnd(d, W)
    q[:, :2], k[:, :2], k[-1] = 0.0, 0.0, 0.0
    q[:, 0], k[:, 1], v[:, 1] = torch.cat([u] * H) * 2.0, u * 2.0, 1.0
    w = {"q": q, "k": k, "v": v, "o": torch.cat([torch.eye(W)[:, :d]] * H, dim=1) * 0.5, "sink": torch.zeros(H)}
    return m, {n: bf(t) for n, t in w.items()}, bf(h)


@pytest.mark.parametrize("dtype,tol", LAYER_BOTH)
@pytest.mark.parametrize("size,key_at", [(32, 40), (32, 47), (30, 20), (33, 15), (30, 0), (2, 63), (64, 127), (100, 3)])
def test_a_marked_key_at_the_edge_of_the_window(size, key_at, dtype, tol):
    """The marked token is seen up to the window's last position and not one further, in a prompt and in decoding. Plain models whose
    window is one off must differ visibly."""
    T, W = 230, 32
    m, w, h = marked_case(T, size, key_at)
    want = plain_attention(h, w, m)[0]
    scale, leaves = np.abs(want).max(), key_at + size
    for other in (size + 1, size - 1):
        got = plain_attention(h, w, dict(m, mask={"size": other}))[0]
        assert np.abs(got - want)[leaves - 2:leaves + 2].max() > 0.2 * scale, f"the case does not show a window of {other}"
    for cuts in ([T], [leaves - 1] + [1] * 20 + [T - leaves - 19], [leaves + 1, 2, T - leaves - 3], [key_at + 1] + [1] * (T - key_at - 1),
                 [leaves, T - leaves]):
        got = with_context(build_attention(m, w, dtype, 16, W=W), h, dtype, 16, cuts)
        close(got, want, tol, f"cuts {cuts[:2]}")


@pytest.mark.parametrize("dtype,tol", LAYER_BOTH)
@pytest.mark.parametrize("sink", [-4.0, 2.0, 40.0])
def test_a_far_key_among_hundreds_and_the_sink(dtype, tol, sink):
    """A marked token near the start of 1,300 under a window that still holds it; sinks that take nothing, some, nearly everything."""
    T, W = 1300, 32
    m, w, h = marked_case(T, 1250, 61)
    w["sink"] = bf(torch.tensor([sink, sink + 1]))
    h[:, 0] = torch.where(torch.arange(T) >= T - 20, 3.0, 0.0)       # only the last queries look for it
    rows = np.concatenate([np.arange(0, 70, 7), np.arange(T - 20, T)])
    f, hh = {k: plain.f64(v) for k, v in w.items()}, plain.f64(bf(h))
    freq, mag = plain.frequencies(m["rot"])
    q, k = (plain.unit_rms(plain.rotate_halves((hh @ f[n].T).reshape(T, -1, 16), freq, mag), EPS) for n in "qk")
    v = (hh @ f["v"].T).reshape(T, 16)
    out = np.zeros((len(rows), 32))
    for i, t in enumerate(rows):
        lo = max(0, t - 1249)
        for a in range(2):
            e = np.exp(k[lo:t + 1, 0] @ q[t, a] * m["scale"])
            out[i, 16 * a:16 * a + 16] = e @ v[lo:t + 1] / (e.sum() + np.exp(f["sink"][a]))
    want = out @ f["o"].T
    for cuts in ([T], [1280] + [1] * 20, [333, 700, 2, 245] + [1] * 20):
        close(with_context(build_attention(m, w, dtype, 64, W=W), bf(h), dtype, 64, cuts).numpy()[rows], want, tol, f"cuts {cuts[:2]}")
    if sink < 0:                              # positions 61 .. 61 + 1249 = 1310 still see the key; a sink of e^40 takes everything
        assert np.abs(want[-20:]).max() > 1
    if sink > 30:
        assert np.abs(want).max() < 0.05


@pytest.mark.parametrize("dtype,tol", LAYER_BOTH)
def test_the_first_tokens_of_a_sequence(dtype, tol):
    """One token alone (its own key and the sink), then two: nothing of what the pages held before is seen."""
    m, w, h = attention_case(4, 2, 24, 16, 8, 16, 9, seed=5)
    want = plain_attention(h, w, m)[0]
    for cuts in ([1, 1, 1, 2, 4], [9], [2, 7], [1, 8]):
        close(with_context(build_attention(m, w, dtype, 16), h, dtype, 16, cuts), want, tol, f"cuts {cuts}")


def test_a_captured_layer_gives_the_eager_result_at_every_replay():
    """The store and attention of single-token steps in a graph, replayed on changing inputs with eager work in between."""
    from nano_vllm_amd.attn_meta import reset_context, set_context
    m, w, _ = attention_case(8, 2, 32, 16, 20, 16, 1, seed=3)
    mix = build_attention(m, w, BF16, 16)
    a = mix.attn
    a.k_cache = torch.zeros(6 * 16, 2, 32, dtype=BF16, device="cuda")
    a.v_cache = torch.zeros(6 * 16, 2, 16, dtype=BF16, device="cuda")
    h, pos, slots = torch.zeros(3, 40, dtype=BF16, device="cuda"), torch.zeros(3, dtype=torch.int64, device="cuda"), torch.zeros(3, dtype=torch.int32, device="cuda")
    bt = torch.arange(6, dtype=torch.int32, device="cuda").view(3, 2).contiguous()
    por = portions([1, 1, 1], [0, 0, 0], [0, 1, 2])
    first = torch.zeros(3, 32, dtype=BF16, device="cuda")
    set_context(True, slot_mapping=slots, block_tables=bt, portions=por)
    try:
        with torch.inference_mode():
            mix(h, pos, [first])
            torch.cuda.synchronize()
            graph = torch.cuda.CUDAGraph()
            with torch.cuda.graph(graph):
                out = mix(h, pos, [first])
            rnd = normal(1)
            for t in range(24):
                h.copy_(bf(rnd(3, 40)))
                first.copy_(bf(rnd(3, 32)))
                pos.fill_(t)
                por.ctx0.fill_(t)
                slots.copy_(torch.tensor([32 * s + t for s in range(3)], dtype=torch.int32))
                graph.replay()
                torch.cuda.synchronize()
                got, kc = out.clone(), a.k_cache.clone()
                assert torch.equal(mix(h, pos, [first]), got) and torch.equal(a.k_cache, kc), f"replay {t}"
    finally:
        reset_context()


# ---------------------------------------------------------------------------------------------- feed-forwards
@pytest.mark.parametrize("dtype,tol", LAYER_BOTH)
@pytest.mark.parametrize("experts,top,ff,shared,n", [(6, 2, 32, 48, 50), (4, 1, 24, 0, 7), (5, 5, 16, 8, 300), (70, 3, 20, 16, 600), (1, 1, 10, 4, 3)])
def test_experts_chosen_by_biased_logits(dtype, tol, experts, top, ff, shared, n):
    """Biases large enough to change choices; the weights are a softmax over the chosen logits, biases included."""
    from nano_vllm_amd import ops_seq
    from nano_vllm_amd.mixers import RoutedExperts
    W = 64
    rnd = normal(experts * 10 + top)
    w = {"router": bf(2 * rnd(experts, W) / W ** 0.5), "router.b": bf(2 * rnd(experts))}
    for e in range(experts):
        w.update({f"e{e}.gate": bf(2 * rnd(ff, W) / W ** 0.5), f"e{e}.up": bf(2 * rnd(ff, W) / W ** 0.5), f"e{e}.down": bf(rnd(W, ff) / ff ** 0.5)})
    if shared:
        w.update({"shared.gate": bf(rnd(shared, W) / W ** 0.5), "shared.up": bf(rnd(shared, W) / W ** 0.5), "shared.down": bf(rnd(W, shared) / shared ** 0.5)})
    mlp = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared} if shared else None}
    h, x, nw, ls = bf(rnd(n, W)), rnd(n, W), bf(1 + 0.1 * rnd(W)), bf(0.5 + 0.1 * rnd(W))
    f = {k: plain.f64(v) for k, v in w.items()}
    want = plain.experts(plain.f64(h), f, mlp)
    if top < experts:
        assert np.abs(plain.experts(plain.f64(h), dict(f, **{"router.b": 0 * f["router.b"]}), mlp) - want).max() > 0.1 * np.abs(want).max()
    mix = build(RoutedExperts, w, dtype, W, experts, ff, top, shared_ff=shared, shared_gate=False, corrected=False, router_bias=True)
    with torch.inference_mode():
        close(mix(dev(h, dtype)), want, tol)
        rows, plan, wts, sh, gate = mix.parts(dev(h, dtype), wide=dev(h.float()))
        assert gate is None and (sh is None) == (not shared)
        res, out = dev(x), torch.empty(n, W, dtype=dtype, device="cuda")
        ops_seq.branch_norm(res, sh, dev(nw, dtype), dev(ls, dtype), EPS, out, (rows, plan, wts))
    close(res, plain.branch(plain.f64(x), want, plain.f64(nw), plain.f64(ls), EPS), tol, "stream")


@pytest.mark.parametrize("dtype,tol", LAYER_BOTH)
@pytest.mark.parametrize("ff,n", [(48, 30), (13, 5), (128, 1)])
def test_gated_feed_forward(dtype, tol, ff, n):
    from nano_vllm_amd.mixers import SiluGLU
    rnd = normal(ff)
    w = {"gate": bf(rnd(ff, 40) / 5), "up": bf(rnd(ff, 40) / 5), "down": bf(rnd(40, ff) / ff ** 0.5)}
    h = bf(rnd(n, 40))
    with torch.inference_mode():
        close(build(SiluGLU, w, dtype, 40, ff)(dev(h, dtype)), plain.gated_unit(plain.f64(h), {k: plain.f64(v) for k, v in w.items()}), tol)


# ---------------------------------------------------------------------------------------------- the engine
def small_config(variant: int) -> dict:
    def att(H, G, d, dv, size, rot, mix, mlp, scale=1.3):
        m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": scale * d ** -0.5, "v_mix": mix}
        if size:
            m["mask"] = {"size": size}
        if rot:
            m["rot"] = rot
        return {"type": "attention", "mixer": m, "mlp": mlp}
    dense = lambda ff: {"kind": "dense", "ff": ff}
    moe = lambda e, top, ff, shared: {"kind": "moe", "router": {"experts": e, "top": top}, "expert": {"ff": ff},
                                      **({"shared": {"ff": shared}} if shared else {})}
    base = {"architecture": "Reselorn", "norm": {"eps": 1e-5}}
    if variant == 0:                                  # a layer that does not mix comes first; all experts are chosen
        return dict(base, vocab=200, width=80, layers=[
            att(2, 1, 16, 40, 30, dict(ROT), False, dense(96)), att(4, 2, 16, 24, 24, dict(ROT), True, moe(3, 3, 16, 0)),
            att(3, 3, 24, 8, 50, dict(ROT, dims=16), False, dense(40)), att(8, 2, 32, 24, 40, dict(ROT, dims=32), True, moe(4, 4, 32, 48))])
    if variant == 1:                                  # choices among many experts, layers without a feed-forward, rotation unscaled or absent
        return dict(base, vocab=150, width=72, layers=[
            att(8, 1, 24, 16, 16, dict(ROT, dims=24, scaling=None), True, moe(12, 2, 24, 8)), att(2, 1, 40, 16, 9, None, True, None),
            att(4, 1, 24, 16, 64, dict(ROT, dims=20, base=5000.0), True, moe(5, 1, 16, 40))])
    return dict(base, vocab=96, width=50, norm={"eps": 1e-3}, layers=[          # nothing divisible by anything, a window of one, no window
        att(3, 3, 9, 21, 1, dict(ROT, dims=6), True, moe(4, 2, 13, 5)), att(6, 3, 10, 21, 0, dict(ROT, dims=10), True, dense(7)),
        att(1, 1, 5, 11, 33, dict(ROT, dims=2), False, None)])


@pytest.fixture(scope="module")
def checkpoints():
    from nano_vllm_amd.reselorn import write_synthetic_checkpoint
    root = tempfile.mkdtemp(prefix="rsl_")
    return [write_synthetic_checkpoint(os.path.join(root, f"m{v}"), small_config(v), seed=51 + v) for v in range(3)]


def engine(path, dtype="float32", pages=40, page=16, live=4, **kw):
    from nano_vllm_amd import LLM
    kw.setdefault("enforce_eager", True)
    kw.setdefault("max_num_batched_tokens", 1024)
    kw.setdefault("max_model_len", 640)
    return LLM(path, dtype=dtype, kvcache_block_size=page, num_kvcache_blocks=pages, max_num_seqs=live, **kw)


def rel(got, want, scale):
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    return float(np.sqrt((d ** 2).mean(-1)).max() / scale)


TOL = {"float32": 5e-5, "bfloat16": 6e-2}


@pytest.mark.parametrize("variant,dtype", [(0, "float32"), (1, "float32"), (2, "float32"), (0, "bfloat16")])
def test_whole_prompt_portions_and_decoding_agree_with_the_plain_model(checkpoints, variant, dtype):
    path = checkpoints[variant]
    ref = plain.Model.load(path)
    toks = torch.randint(0, ref.cfg["vocab"], (150,), generator=torch.Generator().manual_seed(variant)).tolist()
    layers = []
    want = ref.run(toks, layers)
    scale = float(want.std())
    llm = engine(path, dtype)
    try:
        model = llm.model_runner.model
        model.layer_trace = []
        whole = llm.replay_step([{"id": "w", "tokens": toks, "want": list(range(150))}], ["w"])
        seen, model.layer_trace = model.layer_trace, None
        assert len(seen) == len(ref.cfg["layers"])
        for i, x in enumerate(seen):
            close(x, layers[i], 2e-5 if dtype == "float32" else 6e-2, f"residual after layer {i}")
        assert rel(whole, want, scale) <= TOL[dtype]
        # portions of changing size, down to two tokens and single tokens, cut inside pages and windows
        for name, cuts in (("a", [2, 3, 2, 40, 1, 1, 17, 2, 64, 18]), ("b", [149, 1]), ("c", [1] * 60 + [90]), ("d", [2] * 75)):
            at, rows = 0, []
            for c in cuts:
                rows.append(llm.replay_step([{"id": name, "tokens": toks[at:at + c], "want": list(range(c))}],
                                            [name] if at + c == 150 else []))
                at += c
            assert at == 150 and rel(np.concatenate(rows), want, scale) <= TOL[dtype], name
            if dtype == "float32":
                assert rel(np.concatenate(rows), whole, scale) <= 2e-5, "portions against the whole prompt"
        assert llm.scheduler.block_manager.num_free == 40 and llm.scheduler.state_slots.num_free == 4
    finally:
        llm.exit()


@pytest.mark.parametrize("variant,dtype", [(0, "float32"), (1, "float32"), (0, "bfloat16")])
def test_unequal_requests_in_one_batch_equal_each_alone_with_pages_and_slots_reused(checkpoints, variant, dtype):
    """Five requests through four slots and a pool that cannot hold them all at once: prompts in portions beside single tokens
    of others, requests that sit out steps, ends that free pages and slots for the next request."""
    path = checkpoints[variant]
    ref = plain.Model.load(path)
    g = torch.Generator().manual_seed(4)
    lens = {"p": 130, "q": 61, "r": 3, "s": 97, "t": 200}
    toks = {k: torch.randint(0, ref.cfg["vocab"], (n,), generator=g).tolist() for k, n in lens.items()}
    want = {k: ref.run(v) for k, v in toks.items()}
    scale = float(want["p"].std())
    llm = engine(path, dtype, pages=28)                              # 448 token places for 491 tokens
    try:
        plan = [[("p", 50), ("q", 2)], [("p", 1), ("q", 30), ("r", 3)], [("p", 1), ("s", 64)], [("q", 29), ("p", 2), ("s", 1)],
                [("p", 76), ("s", 32)], [("t", 128)], [("t", 2)], [("t", 1)], [("t", 69)]]
        at = {k: 0 for k in lens}
        got = {k: [] for k in lens}
        for step in plan:
            entries, end = [], []
            for k, c in step:
                entries.append({"id": k, "tokens": toks[k][at[k]:at[k] + c], "want": list(range(c))})
                at[k] += c
                if at[k] == lens[k]:
                    end.append(k)
            out = llm.replay_step(entries, end)
            o = 0
            for k, c in step:
                got[k].append(out[o:o + c])
                o += c
        assert at == lens
        for k in lens:
            assert rel(np.concatenate(got[k]), want[k], scale) <= TOL[dtype], k
        assert llm.scheduler.block_manager.num_free == 28 and llm.scheduler.state_slots.num_free == 4
    finally:
        llm.exit()


@pytest.mark.parametrize("page", [16, 64])
def test_long_decoding_across_many_pages(checkpoints, page):
    path = checkpoints[0]
    ref = plain.Model.load(path)
    toks = torch.randint(0, ref.cfg["vocab"], (330,), generator=torch.Generator().manual_seed(8)).tolist()
    want = ref.run(toks)
    llm = engine(path, "float32", pages=384 // page, page=page)
    try:
        rows = [llm.replay_step([{"id": 0, "tokens": toks[:10], "want": list(range(10))}])]
        rows += [llm.replay_step([{"id": 0, "tokens": [t], "want": [0]}]) for t in toks[10:]]
        assert rel(np.concatenate(rows), want, float(want.std())) <= 5e-5
    finally:
        llm.exit()


@pytest.mark.parametrize("eager", [True, False])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_generate_matches_the_plain_model(checkpoints, dtype, eager):
    """LLM.generate() with token-id prompts: scheduler, chunked prefill, block manager, slots, sampler; eagerly and with decode
    steps replayed from captured graphs. Where the plain model's two best logits are a close call the comparison stops."""
    from nano_vllm_amd import SamplingParams
    path = checkpoints[0]
    ref = plain.Model.load(path)
    g = torch.Generator().manual_seed(6)
    prompts = [torch.randint(0, ref.cfg["vocab"], (n,), generator=g).tolist() for n in (5, 70, 31)]
    llm = engine(path, dtype, pages=30, enforce_eager=eager, max_num_batched_tokens=48)      # prompts are prefilled in chunks
    try:
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=24, ignore_eos=True), use_tqdm=False)
        assert eager or llm.model_runner.sgraphs, "decode steps were meant to replay graphs"
        assert llm.scheduler.block_manager.num_free == 30 and llm.scheduler.state_slots.num_free == 4
    finally:
        llm.exit()
    margin = 0.05 if dtype == "float32" else 0.2       # (the sampler reads bf16 logits in both)
    checked = 0
    for prompt, o in zip(prompts, outs):
        gen = o["token_ids"]
        assert len(gen) == 24
        logits = ref.run(prompt + gen[:-1])[len(prompt) - 1:]
        for t, row in zip(gen, logits):
            best = np.sort(row)[-2:]
            if float(best[1] - best[0]) > margin * float(row.std()):
                assert t == int(row.argmax())
                checked += 1
    assert checked >= 30


def test_preemption_recomputes_and_a_sampled_run_repeats_itself(checkpoints):
    from nano_vllm_amd import SamplingParams
    path = checkpoints[1]
    g = torch.Generator().manual_seed(2)
    prompts = [torch.randint(0, 150, (n,), generator=g).tolist() for n in (30, 31, 29, 17)]
    greedy = SamplingParams(temperature=0.0, max_tokens=40, ignore_eos=True)
    outs = []
    for pages in (40, 11):
        llm = engine(path, "float32", pages=pages, max_num_batched_tokens=256, max_model_len=128)
        try:
            outs.append([o["token_ids"] for o in llm.generate(prompts, greedy, use_tqdm=False)])
        finally:
            llm.exit()
    assert outs[0] == outs[1]
    warm = []
    for _ in range(2):
        llm = engine(path, "bfloat16", pages=40, max_num_batched_tokens=256, max_model_len=128)
        try:
            warm.append([o["token_ids"] for o in llm.generate(prompts, SamplingParams(temperature=8.0, max_tokens=16, ignore_eos=True),
                                                               use_tqdm=False)])
        finally:
            llm.exit()
    assert warm[0] == warm[1] and warm[0] != [o[:16] for o in outs[0]]


def test_the_schedule_replayer_as_a_program(checkpoints, tmp_path):
    path = checkpoints[2]
    ref = plain.Model.load(path)
    g = torch.Generator().manual_seed(12)
    a, b = (torch.randint(0, ref.cfg["vocab"], (n,), generator=g).tolist() for n in (90, 41))
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:64], "want": [0, 63]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[64:66], "want": []}, {"id": "b", "tokens": b[:40], "want": [39]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[40:], "want": [0]}, {"id": "a", "tokens": a[66:], "want": [23]}], "end": ["a", "b"]}]
    out = tmp_path / "out"
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", str(out),
                           "--max-tokens", "192"], input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True,
                          timeout=110)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.split("\n") if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    wa, wb = ref.run(a), ref.run(b)
    scale = float(wa.std())
    got = [np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, ref.cfg["vocab"]) for i in range(3)]
    assert rel(got[0], wa[[0, 63]], scale) <= 5e-5 and rel(got[1], wb[[39]], scale) <= 5e-5
    assert rel(got[2], np.stack([wb[40], wa[89]]), scale) <= 5e-5
