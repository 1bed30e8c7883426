"""Ligidra on the GPU against the plain float64 restatement (oracle/ligidra.py): every mechanism alone at the kernel or layer
boundary, then the engine — whole prompts, portions down to two tokens, token-by-token decoding, unequal batches, reused pages
and slots, window and block edges, far keys, sinks, long decoding, greedy generation through LLM.generate(). Configurations and
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

from oracle import ligidra as plain  # noqa: E402

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
EPS = 1e-5
BOTH = [(torch.float32, 3e-6), (torch.bfloat16, 2.0 ** -8)]


def dev(t, dtype=None):
    return t.to("cuda", dtype=dtype or t.dtype).contiguous()


def bf(t):
    return t.to(torch.bfloat16)


def portions(lens, ctx0, slots, max_q=0):
    from nano_vllm_amd.ops_seq import Portions
    cu = np.concatenate([[0], np.cumsum(lens)]).astype(np.int32)
    tseq = np.repeat(np.arange(len(lens)), lens).astype(np.int32)
    i32 = lambda a: torch.tensor(np.asarray(a, dtype=np.int32), device="cuda")
    return Portions(i32(cu), i32(ctx0), i32(slots), i32(tseq), len(lens), int(cu[-1]), max_q or max(lens))


def close(got, want, tol, what=""):
    got = got.double().cpu().numpy() if hasattr(got, "cpu") else np.asarray(got, dtype=np.float64)
    want = want.double().cpu().numpy() if hasattr(want, "cpu") else np.asarray(want, dtype=np.float64)
    err = np.abs(got - want).max() / max(np.abs(want).max(), 1e-9)
    assert err <= tol, f"{what}: relative error {err:.3e} > {tol:.1e}"


# ---------------------------------------------------------------------------------------------- norms, shift, lookups
@pytest.mark.parametrize("dtype,tol", BOTH)
@pytest.mark.parametrize("W", [48, 70, 1, 352, 1536])
@pytest.mark.parametrize("branch", ["none", "plain", "normed"])
def test_shift_norm_adds_norms_and_blends_with_the_previous_token(dtype, tol, W, branch):
    """Two sequences in portions of unequal length (one token, several, the whole rest), state slots full of another sequence's
    rows; what a portion's first row sees of the token before it comes from the slot."""
    from nano_vllm_amd import ops_seq
    g = torch.Generator().manual_seed(W)
    rnd = lambda *s: torch.randn(*s, generator=g)
    T = 12
    xs, As = [rnd(T, W) for _ in range(2)], [bf(rnd(T, W)) for _ in range(2)]
    w, wa, mu = bf(1 + 0.2 * rnd(W)), bf(1 + 0.2 * rnd(W)), bf(torch.rand(W, generator=g))
    f = plain.f64
    ys, hs = [], []
    for x, a in zip(xs, As):
        y = f(x)
        if branch == "plain":
            y = y + f(a)
        elif branch == "normed":
            y = y + plain.norm(f(a), f(wa), EPS)
        ys.append(y)
        hs.append(plain.token_shift(plain.norm(y, f(w), EPS), f(mu)))
    state = torch.full((4, W), 7.0, device="cuda")
    at = [0, 0]
    for lens in ([5, 1], [1, 2], [2, 8], [4, 1]):
        x = dev(torch.cat([xs[i][at[i]:at[i] + n] for i, n in enumerate(lens)]))
        a = dev(torch.cat([As[i][at[i]:at[i] + n] for i, n in enumerate(lens)]), dtype)
        out = torch.empty(sum(lens), W, dtype=dtype, device="cuda")
        y = ops_seq.shift_norm(x, a if branch != "none" else None, dev(wa, dtype) if branch == "normed" else None, dev(w, dtype), dev(mu, dtype), EPS,
                               portions(lens, at, [2, 0]), state, out)
        close(y, np.concatenate([ys[i][at[i]:at[i] + n] for i, n in enumerate(lens)]), 3e-6, "sum")
        close(out, np.concatenate([hs[i][at[i]:at[i] + n] for i, n in enumerate(lens)]), tol, f"portions {lens}")
        at = [p + n for p, n in zip(at, lens)]
    assert bool((state[1] == 7.0).all()) and bool((state[3] == 7.0).all())


@pytest.mark.parametrize("n", [2049, 8200])
def test_shift_norm_with_several_rows_per_workgroup(n):
    """Large steps give a workgroup several consecutive rows: portion borders inside and at the edges of a workgroup's rows."""
    from nano_vllm_amd import ops_seq
    W, g = 40, torch.Generator().manual_seed(n)
    lens = [1, 3, 4, 9, 1, 1, 6, 7]
    lens.append(n - sum(lens))
    x, a = torch.randn(n, W, generator=g), torch.randn(n, W, generator=g)
    w, mu = 1 + 0.2 * torch.randn(W, generator=g), torch.rand(W, generator=g)
    ctx = [0, 5, 0, 8, 3, 0, 16, 2, 0]
    before = torch.randn(len(lens), W, generator=g)
    state = dev(before)
    out = torch.empty(n, W, device="cuda")
    ops_seq.shift_norm(dev(x), dev(a), None, dev(w), dev(mu), EPS, portions(lens, ctx, list(range(len(lens)))), state, out)
    h = plain.norm(plain.f64(x) + plain.f64(a), plain.f64(w), EPS)
    want, at, last = np.zeros_like(h), 0, []
    for i, ln in enumerate(lens):
        prev = np.concatenate([(plain.f64(before[i]) if ctx[i] else np.zeros(W))[None], h[at:at + ln - 1]])
        want[at:at + ln] = h[at:at + ln] + (prev - h[at:at + ln]) * plain.f64(mu)
        at += ln
        last.append(h[at - 1])
    close(out, want, 3e-6)
    close(state, np.stack(last), 3e-6, "state")


@pytest.mark.parametrize("dtype,tol", BOTH)
def test_embedding_norm_gated_lookup_and_rounded_sums(dtype, tol):
    from nano_vllm_amd import ops_seq
    g = torch.Generator().manual_seed(3)
    V, W, D, n = 50, 72, 10, 37
    table, side, w = bf(torch.randn(V, W, generator=g)), bf(torch.randn(V, 4 * D, generator=g)), bf(1 + 0.1 * torch.randn(W, generator=g))
    ids, z, a = torch.randint(0, V, (n,), generator=g), bf(2 * torch.randn(n, D + 3, generator=g)), bf(torch.randn(n, W, generator=g))
    x = torch.empty(n, W, device="cuda")
    ops_seq.embed_norm(dev(table, dtype), dev(ids), dev(w, dtype), EPS, x)
    want = plain.norm(plain.f64(table)[ids.numpy()], plain.f64(w), EPS)
    close(x, want, 3e-6)
    got = ops_seq.gated_lookup(dev(z, dtype)[:, :D], dev(side, dtype), 2 * D, dev(ids))
    close(got, plain.gelu_tanh(plain.f64(z)[:, :D]) * plain.f64(side)[ids.numpy()][:, 2 * D:3 * D], tol)
    out = torch.empty(n, W, dtype=dtype, device="cuda")
    ops_seq.add_group_norm(x, None, 1, EPS, out, dev(a, dtype))       # no weights: the sum itself, rounded
    close(x, want + plain.f64(a), 3e-6)
    close(out, want + plain.f64(a), tol)


@pytest.mark.parametrize("dtype,tol", BOTH)
@pytest.mark.parametrize("W", [4, 260, 1028, 4096, 5000, 8192, 9000])
def test_row_norms_of_wide_rows(dtype, tol, W):
    """Rows that fit a workgroup's registers (one to eight accesses per thread) and one that does not: the norm ahead of a feed-forward,
    the normed embedding, and the last norm on selected rows with a branch that is normed and added only there."""
    from nano_vllm_amd import ops_seq
    g = torch.Generator().manual_seed(W)
    n = 5
    x, a, w, wa = torch.randn(n, W, generator=g), bf(torch.randn(n, W, generator=g)), bf(1 + 0.2 * torch.randn(W, generator=g)), bf(torch.randn(W, generator=g))
    f = plain.f64
    xd, out = dev(x), torch.empty(n, W, dtype=dtype, device="cuda")
    ops_seq.add_group_norm(xd, dev(w, dtype), 1, EPS, out, dev(a, dtype))
    close(xd, f(x) + f(a), 3e-6)
    close(out, plain.norm(f(x) + f(a), f(w), EPS), tol)
    rows = torch.tensor([3, 0, 3], dtype=torch.int32, device="cuda")
    picked, xd = torch.empty(3, W, dtype=dtype, device="cuda"), dev(x)
    ops_seq.offset_norm_rows(xd, rows, 3, dev(w, dtype), EPS, picked, w_off=0.0, a=dev(a, dtype), wa=dev(wa, dtype))
    close(picked, plain.norm(f(x) + plain.norm(f(a), f(wa), EPS), f(w), EPS)[[3, 0, 3]], tol)
    assert torch.equal(xd.cpu(), x), "selected rows are only read"
    ids, emb = torch.tensor([2, 0, 2, 4]), torch.empty(4, W, device="cuda")
    ops_seq.embed_norm(dev(a, dtype), dev(ids), dev(w, dtype), EPS, emb)
    close(emb, plain.norm(f(a)[ids.numpy()], f(w), EPS), 3e-6)


@pytest.mark.parametrize("dtype,tol", BOTH)
@pytest.mark.parametrize("groups,gsz,n", [(4, 64, 5), (6, 128, 70), (5, 256, 3), (7, 20, 9), (4, 130, 4200), (3, 32, 6), (40, 128, 4100)])
@pytest.mark.parametrize("silu", [False, True])
def test_norm_per_head_then_gate(dtype, tol, groups, gsz, n, silu):
    from nano_vllm_amd import ops_seq
    g = torch.Generator().manual_seed(groups * gsz)
    inner = groups * gsz
    y, z, w = torch.randn(n, inner, generator=g), bf(torch.randn(n, inner + 5, generator=g)), bf(1 + 0.2 * torch.randn(gsz, generator=g))
    out = torch.empty(n, inner, dtype=dtype, device="cuda")
    ops_seq.gated_group_norm(dev(y), dev(z, dtype)[:, 5:], dev(w, dtype), groups, EPS, out, norm_first=True, silu=silu)
    zf = plain.f64(z)[:, 5:]
    want = plain.norm(plain.f64(y).reshape(n, groups, gsz), plain.f64(w), EPS).reshape(n, inner) * (plain.silu(zf) if silu else plain.sigmoid(zf))
    close(out, want, tol if dtype == torch.bfloat16 else 1e-5)


@pytest.mark.parametrize("dtype,tol", BOTH)
@pytest.mark.parametrize("taps,C", [(1, 7), (2, 40), (3, 300), (4, 64), (6, 20)])
def test_convolution_of_short_and_long_portions(dtype, tol, taps, C):
    """Steps of short portions walk the taps in registers, long steps take tiles of tokens, others a thread per token: all continue
    from the same state."""
    from nano_vllm_amd import ops_seq
    g = torch.Generator().manual_seed(taps)
    T = 640
    u, w = bf(torch.randn(T, C + 4, generator=g)), bf(torch.randn(C, taps, generator=g))
    want = plain.short_conv(plain.f64(u)[:, :C], plain.f64(w))
    state = torch.full((3, taps - 1, C), 5.0, device="cuda")
    at, rows = 0, []
    for c in (1, 1, 2, 9, 1, 3, 20, 1, 1, 1, 300, 2, 298):
        out = torch.empty(c, C, dtype=dtype, device="cuda")
        ops_seq.causal_conv(dev(u[at:at + c], dtype)[:, :C], dev(w, dtype), None, 1, portions([c], [at], [1]), state, out)
        rows.append(out)
        at += c
    assert at == T
    close(torch.cat(rows), want, tol if dtype == torch.bfloat16 else 1e-5)


# ---------------------------------------------------------------------------------------------- layers in a step's context
def with_context(mixes, h, dtype, block, cuts, path="auto", slot=1):
    """Run `mixes` (a layer, or layers of which later ones may read the first one's cache) on the rows of h in portions `cuts`,
    through pages in scattered order; returns every layer's rows. State slots and summaries start with other content."""
    from nano_vllm_amd import ops_seq
    from nano_vllm_amd.attn_meta import reset_context, set_context
    mixes = mixes if isinstance(mixes, list) else [mixes]
    T = h.shape[0]
    pages = -(-T // block)
    order = torch.randperm(pages + 3, generator=torch.Generator().manual_seed(2))[:pages].to(torch.int32)
    for mod in [m for mix in mixes for m in mix.modules()]:
        if hasattr(mod, "kv_shapes") and mod.kv_shapes() is not None:
            ks, vs = mod.kv_shapes()
            mod.block_size = block
            mod.k_cache = torch.full(((pages + 3) * block, *ks), 2.0, dtype=dtype, device="cuda")
            mod.v_cache = torch.full(((pages + 3) * block, *vs), -2.0, dtype=dtype, device="cuda")
        if hasattr(mod, "page_shapes"):
            for name, shape in mod.page_shapes().items():
                setattr(mod, name, torch.full((pages + 3, *shape), 9.0, dtype=dtype, device="cuda"))
        if hasattr(mod, "state_shapes"):
            for name, shape in mod.state_shapes().items():
                setattr(mod, name, torch.full((3, *shape), 3.0, device="cuda"))
    ops_seq.load_library().nvs_window_attn_force_scalar({"auto": 0, "scalar": 1, "unpacked": 3}.get(path, 0))
    ops_seq.load_library().nvs_delta_force({"walk": 1, "chunks": 2}.get(path, 0))
    outs, at = [[] for _ in mixes], 0
    try:
        with torch.inference_mode():
            for c in cuts:
                pos = torch.arange(at, at + c)
                slots = (order[pos // block].long() * block + pos % block).to(torch.int32)
                set_context(True, slot_mapping=dev(slots), block_tables=dev(order.view(1, -1)), portions=portions([c], [at], [slot]))
                for mix, o in zip(mixes, outs):
                    o.append(mix(dev(h[at:at + c], dtype), dev(pos)).float().cpu())
                at += c
    finally:
        reset_context()
        ops_seq.load_library().nvs_window_attn_force_scalar(0)
        ops_seq.load_library().nvs_delta_force(0)
    assert at == T
    return [torch.cat(o) for o in outs]


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


# ---------------------------------------------------------------------------------------------- attention
ROT = {"dims": 8, "base": 100.0, "scaling": {"factor": 4.0, "low": 1.0, "high": 3.0, "original": 64}}


def attention_case(H, G, d, dv, size, pool, rot_dims, cap, T, seed, W=40, sharp=1.5):
    g = torch.Generator().manual_seed(seed)
    rnd = lambda *s: torch.randn(*s, generator=g)
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": sharp * d ** -0.5, "softcap": cap, "mask": {"size": size, "pool": pool}}
    if rot_dims:
        m["rot"] = dict(ROT, dims=rot_dims)
    w = {"q": rnd(H * d, W) / W ** 0.5, "k": rnd(G * d, W) / W ** 0.5, "v": rnd(G * dv, W) / W ** 0.5, "o": rnd(W, H * dv) / (H * dv) ** 0.5,
         "q.norm": 1 + 0.2 * rnd(H * d), "k.norm": 1 + 0.2 * rnd(G * d), "sink": 1 + rnd(H)}
    return m, {k: bf(v) for k, v in w.items()}, bf(rnd(T, W))


def build_attention(m, w, dtype, block, W=40, source=None):
    from nano_vllm_amd.mixers import AttentionMixer, banded_rotary_frequencies
    rot, mask = m.get("rot"), m.get("mask") or {}
    return build(AttentionMixer, {k: v for k, v in w.items() if source is None or k not in ("k", "v", "k.norm")}, dtype, W, m["heads"],
                 m["kv_heads"], m["dim"], m["vdim"], m["scale"], EPS, block, window=mask.get("size", 0), rot_dims=rot["dims"] if rot else 0,
                 rot_freqs=banded_rotary_frequencies(rot["dims"], rot["base"], rot.get("scaling")) if rot else None, qk_norm=True, bias=False,
                 sink="learned", norm_rows=True, softcap=m.get("softcap") or 0.0, pool=mask.get("pool", 0), source=source)


def plain_attention(h, w, m, kv=None):
    return plain.attention(plain.f64(h), {k: plain.f64(v) for k, v in w.items()}, m, EPS, kv)


CUTS = [[0], [97, 2, 1, 1, 30, 2, 1, 1, 1, 44], [1] * 40 + [2] * 20 + [100]]


@pytest.mark.parametrize("dtype,path,tol", [(torch.float32, "auto", 3e-5), (torch.bfloat16, "auto", 3e-2), (torch.bfloat16, "scalar", 3e-2),
                                            (torch.bfloat16, "unpacked", 3e-2)])
@pytest.mark.parametrize("H,G,d,dv,size,pool,block,rot_dims,cap", [
    (4, 2, 16, 24, 24, 5, 16, 8, 8.0),        # blocks straddle pages
    (8, 1, 24, 16, 7, 3, 32, 24, 30.0),       # eight query heads on one key head; several units of blocks in a page
    (3, 3, 20, 12, 40, 16, 16, 4, 0.0),       # no cap; heads that are no multiple of 8 wide; a block as long as a page
    (2, 1, 64, 80, 1, 1, 16, 0, 5.0),         # a window of one token and blocks of one: every token is seen once
    (1, 1, 40, 40, 33, 50, 16, 16, 12.0),     # blocks longer than the window and than a page
    (6, 2, 136, 72, 16, 8, 64, 40, 20.0),     # long heads
    (2, 2, 16, 200, 500, 4, 48, 16, 9.0),     # a window that nothing leaves
    (20, 2, 8, 8, 50, 2, 64, 8, 6.0),
    # every size of the matrix-core kernels
    (4, 1, 72, 40, 20, 3, 16, 8, 7.0), (2, 2, 128, 128, 30, 6, 32, 64, 20.0), (4, 4, 104, 144, 25, 4, 16, 8, 9.0),
    (2, 1, 192, 64, 18, 5, 16, 16, 11.0), (3, 1, 160, 160, 22, 7, 64, 32, 8.0), (2, 1, 256, 256, 26, 9, 32, 128, 15.0)])
def test_window_with_pooled_blocks_against_the_plain_loop(H, G, d, dv, size, pool, block, rot_dims, cap, dtype, path, tol):
    T = 180
    m, w, h = attention_case(H, G, d, dv, size, pool, rot_dims, cap, T, seed=H * 100 + d)
    want, _ = plain_attention(h, w, m)
    for cuts in CUTS:
        got = with_context(build_attention(m, w, dtype, block), h, dtype, block, [T] if cuts == [0] else cuts, path)[0]
        close(got, want, tol, f"cuts {cuts[:3]}")


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 3e-5), (torch.bfloat16, 3e-2)])
@pytest.mark.parametrize("mask", [{"size": 20, "pool": 6}, {"size": 11, "pool": 4}, {"size": 64, "pool": 9}])
def test_a_layer_that_reads_the_keys_and_values_of_an_earlier_one(dtype, tol, mask):
    """The borrower has queries, window, cap and sinks of its own; blocks of the owner's length are the owner's means, blocks of
    another length are kept by the borrower."""
    T, W = 150, 40
    m, w, h = attention_case(4, 2, 16, 24, 20, 6, 8, 9.0, T, seed=3)
    m2, w2, _ = attention_case(4, 2, 16, 24, mask["size"], mask["pool"], 8, 4.0, T, seed=8)
    want, kv = plain_attention(h, w, m)
    want2, _ = plain_attention(h, {k: v for k, v in w2.items() if k not in ("k", "v", "k.norm")}, m2, kv)
    for cuts in ([T], [70, 2, 1, 1, 1, 33, 1, 41], [1] * 60 + [90]):
        own = build_attention(m, w, dtype, 16)
        bor = build_attention(m2, w2, dtype, 16, source=own)
        assert bor.attn.kv_shapes() is None and bool(bor.attn.page_shapes()) == (mask["pool"] != 6)
        got = with_context([own, bor], h, dtype, 16, cuts)
        close(got[0], want, tol, f"owner, cuts {cuts[:2]}")
        close(got[1], want2, tol, f"borrower, cuts {cuts[:2]}")


def marked_case(T, size, pool, key_at, d=16, W=32, H=2):
    """Every query looks along one direction (its other entries are noise), and the token `key_at` alone has a key along it and a
    value that stands out: wherever it is seen, alone or inside its block, the output shows it."""
    g = torch.Generator().manual_seed(T + key_at)
    m = {"heads": H, "kv_heads": 1, "dim": d, "vdim": d, "scale": 1.0, "softcap": 30.0, "mask": {"size": size, "pool": pool}}
    rnd = lambda *s: torch.randn(*s, generator=g)
    h = 0.3 * rnd(T, W)
    h[:, :2] = 0.0
    h[:, 0] = 3.0
    h[key_at, 1] = 12.0
    u = torch.zeros(d)
    u[0] = 1.0
    q, k, v = 0.02 * rnd(H * d, W), 0.3 * rnd(d, W), 0.3 * rnd(d, W)
    q[:, :2], k[:, :2], k[0] = 0.0, 0.0, 0.0                          # (the other keys have nothing along the direction)
    q[:, 0], k[:, 1], v[:, 1] = torch.cat([u] * H) * 2.0, u * 2.0, 1.0
    w = {"q": q, "k": k, "v": v, "o": torch.cat([torch.eye(W)[:, :d]] * H, dim=1) * 0.5, "q.norm": torch.ones(H * d),
         "k.norm": 8 * torch.ones(d), "sink": torch.zeros(H)}
    return m, {n: bf(t) for n, t in w.items()}, bf(h)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 3e-5), (torch.bfloat16, 3e-2)])
@pytest.mark.parametrize("size,pool,key_at", [(32, 8, 40), (32, 8, 47), (30, 7, 20), (30, 7, 0), (16, 12, 23), (64, 5, 127)])
def test_a_marked_key_at_the_edges_of_the_window_and_of_its_block(size, pool, key_at, dtype, tol):
    """The marked token leaves the window, is not seen at all until its whole block has left, and is then seen as a part of the
    block's mean — in a prompt and in decoding. Plain models whose window or block is one off must differ visibly."""
    T, W = 260, 32
    m, w, h = marked_case(T, size, pool, key_at)
    want, _ = plain_attention(h, w, m)
    scale = np.abs(want).max()
    leaves, block_seen = key_at + size, (key_at // pool + 1) * pool - 1 + size
    for change in ({"size": size + 1}, {"size": size - 1}, {"pool": pool + 1}, {"pool": pool - 1}):
        other, _ = plain_attention(h, w, dict(m, mask=dict(m["mask"], **change)))
        assert np.abs(other - want)[leaves - 2:block_seen + 3].max() > 0.02 * scale, f"the case does not show {change}"
    cuts = ([T], [leaves - 1] + [1] * (T - leaves + 1), [leaves + 1, 2, 2] + [1] * 20 + [T - leaves - 25], [block_seen, 2, T - block_seen - 2])
    for c in cuts:
        got = with_context(build_attention(m, w, dtype, 16, W=W), h, dtype, 16, c)[0]
        close(got, want, tol, f"cuts {c[:2]}")


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 3e-5), (torch.bfloat16, 3e-2)])
def test_a_far_block_among_hundreds_and_the_sink(dtype, tol):
    """A marked token near the start of 1,500, seen only through its block's mean among hundreds of blocks (many rounds of blocks, units
    in many pages); then sinks so large that they take nearly everything."""
    T, W = 1500, 32
    m, w, h = marked_case(T, 48, 4, 61)
    h[:, 0] = torch.where(torch.arange(T) >= T - 20, 3.0, 0.0)       # only the last queries look for it
    h = bf(h)
    for sink in (-3.0, 40.0):
        w["sink"] = bf(torch.full((2,), sink))
        hh = plain.f64(h)
        rows = np.concatenate([np.arange(100), np.arange(700, 740), np.arange(T - 20, T)])
        f = {k: plain.f64(v) for k, v in w.items()}
        q = plain.norm(hh @ f["q"].T, f["q.norm"], EPS).reshape(T, 2, 16)
        k, v = plain.norm(hh @ f["k"].T, f["k.norm"], EPS).reshape(T, 1, 16), (hh @ f["v"].T).reshape(T, 1, 16)
        want = np.stack([plain_row(q[t], k[:t + 1], v[:t + 1], m, f["sink"]) for t in rows]) @ f["o"].T
        for cuts in ([T], [1480] + [1] * 20, [333, 800, 2, 345] + [1] * 20):
            got = with_context(build_attention(m, w, dtype, 64, W=W), h, dtype, 64, cuts)[0].numpy()[rows]
            close(got, want, tol, f"sink {sink}, cuts {cuts[:2]}")
        far = np.abs(want[-20:]).max()
        assert far < 0.01 if sink > 0 else far > 1, far               # (capped scores stay below 30)


def plain_row(q, k, v, m, sink):
    """One query row (the last of k's positions) of the pooled attention, for long sequences."""
    t, size, pool, cap = k.shape[0] - 1, m["mask"]["size"], m["mask"]["pool"], m["softcap"]
    nb = max(0, (t - size + 1) // pool)
    ks = np.concatenate([k[:nb * pool, 0].reshape(nb, pool, k.shape[2]).mean(1), k[max(0, t - size + 1):, 0]])
    vs = np.concatenate([v[:nb * pool, 0].reshape(nb, pool, v.shape[2]).mean(1), v[max(0, t - size + 1):, 0]])
    out = []
    for a in range(q.shape[0]):
        s = cap * np.tanh(ks @ q[a] * m["scale"] / cap)
        e = np.exp(s)
        out.append(e @ vs / (e.sum() + math.exp(sink[a])))
    return np.concatenate(out)


# ---------------------------------------------------------------------------------------------- the delta rule
def delta_case(H, G, d, dv, taps, channelwise, T, seed, W=40, rate=-1.0, dt=-2.0, ranks=(12, 20)):
    g = torch.Generator().manual_seed(seed)
    rnd = lambda *s: torch.randn(*s, generator=g)
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "conv": taps}
    w = {"q": rnd(G * d, W) / W ** 0.5, "k": rnd(G * d, W) / W ** 0.5, "v": rnd(H * dv, W) / W ** 0.5, "o": rnd(W, H * dv) / (H * dv) ** 0.5,
         "q.conv": rnd(G * d, taps) / taps ** 0.5, "k.conv": rnd(G * d, taps) / taps ** 0.5, "v.conv": rnd(H * dv, taps) / taps ** 0.5,
         "b": 2 * rnd(H, W) / W ** 0.5, "A_log": rate + 0.5 * rnd(H), "norm": 1 + 0.2 * rnd(dv), "dt_bias": dt + rnd(H * d if channelwise else H)}
    if channelwise:
        w.update({"a1": rnd(ranks[0], W) / W ** 0.5, "a2": rnd(H * d, ranks[0]) / ranks[0] ** 0.5, "g1": rnd(ranks[1], W) / W ** 0.5,
                  "g2": 2 * rnd(H * dv, ranks[1]) / ranks[1] ** 0.5})
    else:
        w.update({"a": rnd(H, W) / W ** 0.5, "g": rnd(H * dv, W) / W ** 0.5})
    return m, {k: bf(v) for k, v in w.items()}, bf(rnd(T, W))


def build_delta(m, w, dtype, W=40):
    from nano_vllm_amd.mixers import DeltaMixer
    return build(DeltaMixer, w, dtype, W, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], EPS,
                 w["a1"].shape[0] if "a1" in w else 0, w["g1"].shape[0] if "g1" in w else 0)


@pytest.mark.parametrize("dtype,path,tol", [(torch.float32, "auto", 5e-5), (torch.float32, "walk", 5e-5), (torch.float32, "chunks", 5e-5),
                                            (torch.bfloat16, "auto", 5e-2)])
@pytest.mark.parametrize("channelwise", [False, True])
@pytest.mark.parametrize("H,G,d,dv,taps", [(4, 2, 16, 24, 3), (3, 1, 20, 40, 2), (2, 2, 64, 8, 4), (1, 1, 7, 5, 1), (6, 3, 40, 144, 5), (2, 1, 128, 64, 4),
                                           (1, 1, 150, 20, 2)])
def test_delta_rule_against_the_plain_loop(H, G, d, dv, taps, channelwise, dtype, path, tol):
    """Whole prompts, portions that end inside a chunk of tokens, single tokens through a dirty slot; sizes that fill no tile, shared
    query / key heads, key sizes of every kernel size."""
    T = 77
    m, w, h = delta_case(H, G, d, dv, taps, channelwise, T, seed=H * 100 + d)
    want = plain.delta(plain.f64(h), {k: plain.f64(v) for k, v in w.items()}, m, EPS, channelwise)
    for cuts in ([T], [33, 2, 1, 1, 16, 1, 2, 21], [1] * 20 + [57]):
        close(with_context(build_delta(m, w, dtype), h, dtype, 16, cuts, path)[0], want, tol, f"cuts {cuts[:3]}")


@pytest.mark.parametrize("path", ["auto", "walk"])
@pytest.mark.parametrize("channelwise", [False, True])
@pytest.mark.parametrize("rate,dt", [(3.0, 1.0), (1.0, 2.0), (-6.0, -4.0)])
def test_delta_rule_with_decays_that_forget_or_keep_everything(channelwise, rate, dt, path):
    """Decays whose product over a chunk of tokens underflows (every step forgets nearly everything), is small, or keeps the state for
    good over 400 tokens."""
    T = 400 if rate < 0 else 120
    m, w, h = delta_case(2, 1, 24, 20, 3, channelwise, T, seed=5, rate=rate, dt=dt)
    want = plain.delta(plain.f64(h), {k: plain.f64(v) for k, v in w.items()}, m, EPS, channelwise)
    for cuts in ([T], [50, 1, 17, T - 68]):
        close(with_context(build_delta(m, w, torch.float32), h, torch.float32, 16, cuts, path)[0], want, 1e-4, f"cuts {cuts[:2]}")


def test_delta_rule_with_repeated_keys_and_full_steps():
    """The same key over and over with beta near 1: the triangular system of a chunk has entries near one everywhere."""
    T, W = 90, 40
    m, w, h = delta_case(2, 2, 16, 24, 1, False, T, seed=9, rate=-5.0, dt=-4.0)
    h = bf(h.float() * 0.1 + torch.randn(W, generator=torch.Generator().manual_seed(1)))
    w["b"] = bf(w["b"].float() + h.float().mean(0) * 0.3)
    want = plain.delta(plain.f64(h), {k: plain.f64(v) for k, v in w.items()}, m, EPS, False)
    for path in ("chunks", "walk"):
        close(with_context(build_delta(m, w, torch.float32), h, torch.float32, 16, [T], path)[0], want, 2e-4, path)


@pytest.mark.parametrize("channelwise", [False, True])
def test_delta_rule_on_unequal_portions_of_one_step(channelwise):
    """Five sequences in one call — long, one token, two tokens, fresh and continued — equal each alone (walked token by token)."""
    from nano_vllm_amd import ops_seq
    H, G, d, dv = 3, 1, 32, 48
    g = torch.Generator().manual_seed(4)
    rnd = lambda *s: torch.randn(*s, generator=g, device="cpu").cuda()
    lens, ctx, slots = [100, 1, 2, 16, 37], [0, 9, 0, 3, 8], [4, 0, 2, 1, 3]
    n = sum(lens)
    qkv, gates = rnd(n, 2 * G * d + H * dv), rnd(n, 2 * H)
    decays = rnd(n, H * d) if channelwise else None
    A, dt = rnd(H) - 1.0, (rnd(H * d) if channelwise else rnd(H)) - 1.0
    S0 = 0.3 * rnd(5, H, dv, d)

    def run(mode, which):
        S, outs = S0.clone(), []
        cu = np.concatenate([[0], np.cumsum(lens)])
        ops_seq.load_library().nvs_delta_force(mode)
        try:
            for group in which:
                rows = torch.cat([torch.arange(cu[i], cu[i + 1]) for i in group]).cuda()
                por = portions([lens[i] for i in group], [ctx[i] for i in group], [slots[i] for i in group])
                y = torch.empty(por.n, H * dv, device="cuda")
                ops_seq.delta_scan(qkv[rows].contiguous(), gates[rows].contiguous(), H, 0, decays[rows].contiguous() if channelwise else None, A, dt,
                                   d ** -0.5, H, G, d, dv, por, S, y)
                outs.append(y)
        finally:
            ops_seq.load_library().nvs_delta_force(0)
        return torch.cat(outs), S
    y1, s1 = run(1, [[i] for i in range(5)])
    for mode, which in ((0, [list(range(5))]), (2, [list(range(5))]), (2, [[i] for i in range(5)])):
        y, s = run(mode, which)
        close(y, y1, 2e-5)
        close(s, s1, 2e-5, "state")


# ---------------------------------------------------------------------------------------------- experts
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 3e-5), (torch.bfloat16, 3e-2)])
@pytest.mark.parametrize("experts,top,ff,shared,n", [(6, 2, 32, 48, 50), (4, 1, 24, 0, 7), (5, 5, 16, 8, 300), (70, 3, 20, 16, 600)])
def test_routed_experts_with_scores_as_weights_added_to_the_residual(dtype, tol, experts, top, ff, shared, n):
    from nano_vllm_amd.mixers import RoutedExperts
    W = 64
    g = torch.Generator().manual_seed(experts * 10 + top)
    rnd = lambda *s: torch.randn(*s, generator=g)
    w = {"router": bf(4 * rnd(experts, W) / W ** 0.5)}
    for e in range(experts):
        w.update({f"e{e}.gate": bf(2 * rnd(ff, W) / W ** 0.5), f"e{e}.up": bf(2 * rnd(ff, W) / W ** 0.5), f"e{e}.down": bf(rnd(W, ff) / ff ** 0.5)})
    if shared:
        w.update({"shared.gate": bf(rnd(shared, W) / W ** 0.5), "shared.up": bf(rnd(shared, W) / W ** 0.5), "shared.down": bf(rnd(W, shared) / shared ** 0.5)})
    mlp = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared} if shared else None}
    h, x = bf(rnd(n, W)), rnd(n, W)
    want = plain.experts(plain.f64(h), {k: plain.f64(v) for k, v in w.items()}, mlp)
    mix = build(RoutedExperts, w, dtype, W, experts, ff, top, shared_ff=shared, renorm=False, shared_gate=False, corrected=False)
    with torch.inference_mode():
        close(mix(dev(h, dtype)), want, tol)
        res = dev(x)
        out = mix(dev(h, dtype), res=res)
    close(res, want + plain.f64(x), tol, "residual")
    assert out.dtype == dtype and torch.equal(out, res.to(dtype))


# ---------------------------------------------------------------------------------------------- the engine
def small_config(variant: int) -> dict:
    def att(H, G, d, dv, size, pool, rot, cap, mlp, kv_from=None):
        m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": 1.3 * d ** -0.5, "softcap": cap, "mask": {"size": size, "pool": pool}}
        if rot:
            m["rot"] = rot
        if kv_from is not None:
            m["kv_from"] = kv_from
        return {"type": "attention", "mixer": m, "mlp": mlp}

    def dl(H, G, d, dv, taps, mlp, ranks=None):
        m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "conv": taps}
        if ranks:
            m.update(decay_rank=ranks[0], gate_rank=ranks[1])
        return {"type": "channel_delta" if ranks else "delta", "mixer": m, "mlp": mlp}
    moe = lambda e, top, ff, shared: {"kind": "moe", "router": {"experts": e, "top": top}, "expert": {"ff": ff},
                                      **({"shared": {"ff": shared}} if shared else {})}
    base = {"architecture": "Ligidra", "norm": {"eps": 1e-5}}
    if variant == 0:
        return dict(base, vocab=200, width=80, token_side={"dim": 12}, layers=[
            dl(4, 2, 16, 24, 3, moe(3, 3, 32, 48), (10, 14)), att(4, 2, 16, 24, 24, 5, dict(ROT), 8.0, moe(3, 3, 16, 0)),
            dl(2, 1, 24, 16, 4, moe(2, 2, 24, 16)), att(4, 2, 16, 24, 40, 5, dict(ROT), 12.0, moe(3, 3, 32, 48), kv_from=1)])
    if variant == 1:                                  # attention first, choices among many experts, layers without a feed-forward
        return dict(base, vocab=150, width=72, token_side={"dim": 7}, layers=[
            att(8, 1, 24, 16, 16, 3, dict(ROT, dims=24, scaling=None), None, moe(12, 2, 24, 8)), dl(3, 3, 20, 12, 2, None),
            att(2, 1, 24, 16, 9, 7, dict(ROT, dims=24, scaling=None), 6.0, None, kv_from=0), dl(1, 1, 40, 40, 5, moe(5, 1, 16, 40), (6, 30))])
    return dict(base, vocab=96, width=50, norm={"eps": 1e-3}, layers=[          # no side table, nothing divisible by anything
        dl(3, 1, 9, 21, 1, moe(4, 2, 13, 0), (5, 3)), att(3, 3, 10, 6, 1, 2, None, 5.0, None), dl(1, 1, 5, 11, 6, moe(1, 1, 10, 10))])


@pytest.fixture(scope="module")
def checkpoints():
    from nano_vllm_amd.ligidra import write_synthetic_checkpoint
    root = tempfile.mkdtemp(prefix="lgd_")
    return [write_synthetic_checkpoint(os.path.join(root, f"m{v}"), small_config(v), seed=41 + v) for v in range(3)]


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


def test_caches_states_and_summaries_that_the_engine_gives_the_layers(checkpoints):
    from nano_vllm_amd.ligidra import tensor_shapes
    for v, path in enumerate(checkpoints):
        llm = engine(path)
        try:
            model = llm.model_runner.model
            assert set(model.named_loaders()) == set(tensor_shapes(small_config(v)))
            if v == 0:
                own, bor = model.layers[1].mixer.attn, model.layers[3].mixer.attn
                assert bor.k_cache is None and bor.pool_k is None and bor.owner is own and own.k_cache.shape == (640, 2, 16)
                assert own.pool_k.shape == (40, 8, 2, 16) and own.pool_v.shape == (40, 1, 2, 24, 8)
                assert model.layers[0].mixer.rec_state.shape == (5, 4, 24, 16) and model.layers[0].norm1.shift_state.shape == (5, 80)
                assert model.layers[0].mixer.a_rank == 10 and model.layers[0].mixer.g_rank == 14
            if v == 1:
                bor = model.layers[2].mixer.attn
                assert bor.k_cache is None and bor.pool_k.shape == (40, 8, 1, 24)      # blocks of another length: its own means
        finally:
            llm.exit()


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
        if dtype == "float32":                                       # layer by layer, in 32-bit
            for i, x in enumerate(seen):
                close(x, layers[i], 2e-5, f"residual after layer {i}")
        assert rel(whole, want, scale) <= TOL[dtype]
        # portions of changing size, down to two tokens and single tokens, cut inside pages, blocks and chunks
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


@pytest.mark.parametrize("variant", [0, 1])
def test_unequal_requests_in_one_batch_equal_each_alone_with_pages_and_slots_reused(checkpoints, variant):
    """Five requests through four slots and a pool that cannot hold them all at once: prompts in portions beside single tokens
    of others, requests that sit out steps, ends that free pages and slots for the next request."""
    path = checkpoints[variant]
    ref = plain.Model.load(path)
    g = torch.Generator().manual_seed(4)
    lens = {"p": 130, "q": 61, "r": 3, "s": 97, "t": 200}
    toks = {k: torch.randint(0, ref.cfg["vocab"], (n,), generator=g).tolist() for k, n in lens.items()}
    want = {k: ref.run(v) for k, v in toks.items()}
    scale = float(want["p"].std())
    llm = engine(path, "float32", pages=28)                          # 448 token places for 491 tokens
    try:
        plan = [[("p", 50), ("q", 2)], [("p", 1), ("q", 30), ("r", 3)], [("p", 1), ("s", 64)], [("q", 29), ("p", 2), ("s", 1)],
                [("p", 76), ("s", 32)], [("t", 128)], [("t", 2)], [("t", 1)], [("t", 69)]]
        at = {k: 0 for k in lens}
        got = {k: [] for k in lens}
        used_slots = {}
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
            for k, _ in step:
                if k in llm._replay:
                    used_slots[k] = llm._replay[k].state_slot
        assert at == lens
        for k in lens:
            assert rel(np.concatenate(got[k]), want[k], scale) <= 5e-5, k
        assert used_slots["s"] == 2 and used_slots["t"] == 0, "freed slots are handed out again, lowest first"
        assert llm.scheduler.block_manager.num_free == 28 and llm.scheduler.state_slots.num_free == 4
    finally:
        llm.exit()


def test_long_decoding_across_many_pages_and_blocks(checkpoints):
    path = checkpoints[0]
    ref = plain.Model.load(path)
    toks = torch.randint(0, ref.cfg["vocab"], (330,), generator=torch.Generator().manual_seed(8)).tolist()
    want = ref.run(toks)
    llm = engine(path, "float32", pages=24)
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
                          timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.split("\n") if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    wa, wb = ref.run(a), ref.run(b)
    scale = float(wa.std())
    got = [np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, ref.cfg["vocab"]) for i in range(3)]
    assert rel(got[0], wa[[0, 63]], scale) <= 5e-5 and rel(got[1], wb[[39]], scale) <= 5e-5
    assert rel(got[2], np.stack([wb[40], wa[89]]), scale) <= 5e-5
