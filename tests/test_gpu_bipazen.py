"""The Bipazen design on the GPU against its plain implementation: every new kernel alone (across cuts, at odd sizes, with a
key that stands out), then the engine under every cutting in both precisions, tight pools, slots used again, long decoding,
recorded steps, other sizes, models drawn at random, generation through the scheduler, the trace replay and the command line."""
import json
import os
import random
import subprocess
import sys

import numpy as np
import pytest

from tests import helpers as H
from tests.plain import bipazen_plain as P

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
SHAPES = ("bipazen-tiny-a", "bipazen-tiny-b")
LENGTHS = [1, 19, 45, 80, 131]
TOL = {"float32": 1e-9, "bfloat16": 2e-2}     # float32 is the sharp test


def sharpen(folder):
    """Larger query, latent and router matrices, so that few keys carry a row's softmax and experts are told apart; decays near
    one, so that a lost state shows far behind."""
    from safetensors import safe_open
    from safetensors.torch import save_file
    path = os.path.join(folder, "model.safetensors")
    with safe_open(path, framework="pt") as f:
        tensors = {name: f.get_tensor(name) for name in f.keys()}
    for name, t in tensors.items():
        if name.endswith((".mix.q", ".mix.uk", ".mix.dkv", ".mlp.router")):
            tensors[name] = (t.float() * 8.0).to(t.dtype)
        elif name.endswith(".mix.lam"):
            tensors[name] = (t.float() - 5.0).to(t.dtype)
        elif name.endswith(".mix.A_log"):
            tensors[name] = (t.float() - 3.0).to(t.dtype)
    save_file(tensors, path)
    return folder


def write_model(path, cfg, seed, dtype):
    from kipp_amd.weights import write_random_model
    return sharpen(write_random_model(str(path), cfg, seed=seed, dtype=dtype))


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    from kipp_amd.config import shape_config
    root = tmp_path_factory.mktemp("bipazen")
    return {(shape, dtype): write_model(root / f"{shape}-{dtype}", shape_config(shape), 60 + i, dtype)
            for i, shape in enumerate(SHAPES) for dtype in ("float32", "bfloat16")}


_plain_cache = {}
_margin_cache = {}


def plain_logits(folder, tokens):
    key = (folder, tuple(tokens))
    if key not in _plain_cache:
        cfg, w = P.load_folder(folder)
        margins = []
        _plain_cache[key] = P.forward_whole(cfg, w, list(tokens), margins=margins)
        _margin_cache[id(_plain_cache[key])] = np.min(np.array(margins).reshape(-1, len(tokens)), axis=0) if margins else None
    return _plain_cache[key]


FLIPS = 0.5         # share of a request's positions that may lie beyond the bfloat16 bound (see `close`)
CLOSE_CALL = 0.02   # a router's margin (in scores) below which bfloat16 rows may choose another expert


def close(got, ref, tol, what):
    """Every position's normalised squared error within `tol`.  Under the bfloat16 bound a router's choice between two experts
    whose scores differ by less than the rounding of the rows it reads falls either way, and the position (and, through the
    states and keys, every one after it) then differs by much more than rounding: a request passes if every position beyond
    the bound stands at or behind a close call of the plain implementation's routers, or if no more than a share of its
    positions lie beyond it.  The float32 runs of the same cases allow no such position."""
    assert got.shape == ref.shape and np.isfinite(got).all(), what
    each = [float(np.sum((g - r) ** 2) / np.sum(r ** 2)) for g, r in zip(got.astype(np.float64), ref)]
    spared = int(FLIPS * len(each)) if tol >= TOL["bfloat16"] else 0
    margins = _margin_cache.get(id(ref)) if spared else None
    if margins is not None and len(margins) == len(each):
        called = np.minimum.accumulate(margins) < CLOSE_CALL
        if all(e <= tol or c for e, c in zip(each, called)):
            return
    worst = sorted(each)[len(each) - 1 - spared]
    over = sum(e > tol for e in each)
    assert worst <= tol, f"{what}: NMSE {worst:.3e} exceeds {tol:.1e} ({over} of {len(each)} positions beyond it, {spared} spared)"


def engine_of(folder, dtype, page=16, **kw):
    from kipp_amd.engine import Engine
    kw.setdefault("max_tokens", 1024)
    return Engine.from_folder(folder, dtype=dtype, page_size=page, share_prefixes=False, **kw)


def dev(a, ty=None):
    import torch
    return None if a is None else torch.tensor(np.asarray(a), device="cuda:0", dtype=ty)


def f32(a):
    import torch
    return dev(np.asarray(a, dtype=np.float32), torch.float32)


def i32(a):
    import torch
    return dev(np.asarray(a, dtype=np.int32), torch.int32)


def rounded(a, dtype):
    """The values as a tensor of that type holds them, in float64."""
    import torch
    a = np.asarray(a, dtype=np.float32)
    return a.astype(np.float64) if dtype == "float32" else torch.tensor(a).to(torch.bfloat16).double().numpy()


def requests_of(vocab, seed=0, lengths=LENGTHS):
    return {f"r{i}": H.random_tokens(seed * 100 + i, n, vocab) for i, n in enumerate(lengths)}


def _entries(lengths, slots):
    starts = np.concatenate([[0], np.cumsum(lengths)[:-1]])
    seq_of = np.concatenate([np.full(n, i) for i, n in enumerate(lengths)])
    return i32(starts), i32(lengths), i32(slots), i32(seq_of), starts


# =============================================================================== the kernels alone

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width, blocks, taps", [(96, 3, 4), (80, 2, 2), (64, 8, 7), (72, 1, 1), (30, 5, 3), (512, 2, 4), (600, 1, 5), (40, 5, 16), (24, 24, 2),
                                                 (264, 1, 3)])
def test_recurrence_kernels_across_cuts(dtype, width, blocks, taps):
    """Eighteen entries of unequal length in slots of any order: a first portion, a token each (single tokens alone: the one
    launch where the matrices allow it), the rest as portions beside single tokens; from the kept states and filter inputs,
    against the plain functions over the whole sequences.  The matrices are in the model's type, everything else is 32-bit:
    under bfloat16 the result is as exact as under float32, up to the matrices' own rounding.  The slots end at what the
    plain recurrence and filter leave."""
    import torch
    from kipp_amd.csrc import ops
    ty = torch.float32 if dtype == "float32" else torch.bfloat16
    rng = np.random.default_rng(width * 10 + taps)
    size = width // blocks
    y_b, x_b, conv_b = (rng.normal(size=width).astype(np.float32) * 0.3 for _ in range(3))
    conv = rng.normal(size=(width, taps)).astype(np.float32) * 0.5
    ra, ri = (rounded(rng.normal(size=(blocks, size, size)) * (1.5 / np.sqrt(size)), dtype) for _ in range(2))
    ra_b, ri_b = (rng.normal(size=(blocks, size)).astype(np.float32) for _ in range(2))
    lam = (rng.normal(size=width) - 4.0).astype(np.float32)
    decay = f32(8.0 * np.log1p(np.exp(lam.astype(np.float64))))
    mfma = ops.recurrence_mfma_ok(ty, size)
    assert mfma == (dtype == "bfloat16" and size % 8 == 0)
    gates = dev(np.stack([ra, ri], axis=1) if mfma else np.concatenate([ra, ri], axis=1).transpose(0, 2, 1).copy(), ty)
    n = 18
    totals = [int(v) for v in rng.integers(3, 24, size=n - 2)] + [150, 71]
    first = [int(v) for v in rng.integers(1, 3, size=n - 2)] + [100, 70]
    seqs = [rng.normal(size=(t, 2 * width + 5)).astype(np.float32) for t in totals]
    slots = list(rng.permutation(n + 2)[:n])
    state = torch.zeros((n + 2, ops.recurrence_state_size(width, taps)), device="cuda:0")
    got = [[] for _ in totals]
    w = (f32(y_b), f32(x_b), f32(conv.T.copy()), f32(conv_b))
    rb, ib = f32(ra_b.reshape(-1)), f32(ri_b.reshape(-1))
    at = [0] * n
    for part in range(4):
        lengths = [first[i] if part == 0 else (1 if part in (1, 2) or i % 3 == 0 else totals[i] - at[i]) for i in range(n)]
        lengths = [min(l, totals[i] - at[i]) for i, l in enumerate(lengths)]
        live = [i for i in range(n) if lengths[i] > 0]
        proj = f32(np.concatenate([seqs[i][at[i]:at[i] + lengths[i]] for i in live]))
        qs, ql, sl, seq_of, starts = _entries([lengths[i] for i in live], [slots[i] for i in live])
        positions = i32(np.concatenate([np.arange(at[i], at[i] + lengths[i]) for i in live]))
        rows = proj.shape[0]
        out = torch.empty((rows, width), device="cuda:0")
        if part in (1, 2) and mfma:
            ops.recurrence_step(proj, 0, width + 2, *w, gates, rb, ib, decay, state, positions, seq_of, sl, out)
        else:
            u = ops.recurrence_filter(proj, width + 2, w[1], w[2], w[3], state, positions, seq_of, qs, ql, sl, torch.empty((rows, width), device="cuda:0"))
            terms = ops.recurrence_gates(u, gates, rb, ib, decay, torch.empty((rows, width, 2), device="cuda:0"), mfma)
            ops.recurrence_scan(terms, proj, 0, w[0], state, qs, ql, sl, out)
        out = out.cpu().numpy()
        for j, i in enumerate(live):
            got[i].append(out[starts[j]:starts[j] + lengths[i]])
            at[i] += lengths[i]
    for i in range(n):
        s = seqs[i][:at[i]].astype(np.float64)
        x = s[:, width + 2:2 * width + 2] + x_b
        u = P.causal_filter(x, conv, conv_b)
        r, g = P.block_gates(u, ra, ra_b, ri, ri_b)
        S, last = P.gated_recurrence(u, r, g, lam)
        ref = S * P.gelu_tanh(s[:, :width] + y_b)
        out = np.concatenate(got[i])
        assert np.allclose(out, ref, rtol=2e-5, atol=2e-5 * np.abs(ref).max()), (i, np.abs(out - ref).max(), np.abs(ref).max())
        kept = state[slots[i]].cpu().numpy()
        assert np.allclose(kept[:width], last, rtol=2e-5, atol=2e-5 * np.abs(S).max())
        ring = kept[width:width * (1 + taps)].reshape(taps, width)
        for p in range(max(0, at[i] - taps), at[i]):
            assert np.allclose(ring[p % taps], x[p], atol=1e-6), (i, p)
    free = [s for s in range(n + 2) if s not in slots]
    assert float(state[free].abs().max()) == 0.0


def test_recurrence_is_exact_where_the_decay_is_nearly_one():
    """log a of a millionth: 1 - a^2 is taken from the logarithm, not from a rounded a; and a gate that is shut stops the state."""
    import torch
    from kipp_amd.csrc import ops
    width = 16
    u = f32(np.full((3, width), 2.0))
    decay = f32(np.geomspace(1e-7, 50.0, width))
    zero = torch.zeros((1, 2, width, width), dtype=torch.bfloat16, device="cuda:0")
    for bias in (0.0, -80.0, 80.0):
        terms = ops.recurrence_gates(u, zero, f32(np.full(width, bias)), f32(np.zeros(width)), decay, torch.empty((3, width, 2), device="cuda:0"), True)
        r = 1.0 / (1.0 + np.exp(-bias))
        log_a = -r * decay.cpu().numpy().astype(np.float64)
        got = terms.cpu().numpy()
        assert np.allclose(got[1, :, 0], np.exp(log_a), rtol=1e-6)
        assert np.allclose(got[1, :, 1], np.sqrt(-np.expm1(2 * log_a)), rtol=1e-5, atol=1e-12)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("experts, top, tokens, width, inner", [(6, 2, 37, 64, 96), (4, 1, 300, 32, 64), (8, 8, 1, 96, 40), (3, 2, 21, 40, 30), (1, 1, 5, 64, 32),
                                                               (40, 4, 5, 288, 160), (130, 3, 64, 64, 200), (4, 2, 400, 128, 72)])
def test_gated_experts_with_weighed_inputs(dtype, experts, top, tokens, width, inner):
    """Sigmoid scores as weights, not renormalized, on the experts' inputs: choice with ties, the weights in the order of the
    sorted rows, both products with the activation in between (tiles of 16 rows and of 128 on the matrix cores), the sum
    without weights; against loops over tokens.  And the same experts without weights."""
    import torch
    from kipp_amd.csrc import ops
    ty = torch.float32 if dtype == "float32" else torch.bfloat16
    rng = np.random.default_rng(experts * 10 + top)
    z = rng.normal(size=(2, tokens, experts + 3)).astype(np.float32) * 2
    if tokens > 2:
        z[:, 2, :] = 0.0                        # every score equal: the lowest indices
    x = rounded(rng.normal(size=(tokens, width)), dtype)
    w = {}
    for e in range(experts):
        for name, shape in (("gate", (inner, width)), ("up", (inner, width)), ("down", (width, inner))):
            w[f"e{e}.{name}"] = rounded(rng.normal(size=shape) * (2.0 / np.sqrt(shape[1])), dtype)
    pairs = tokens * top
    chosen, weight = torch.empty((tokens, top), dtype=torch.int32, device="cuda:0"), torch.empty((tokens, top), device="cuda:0")
    pair_token, place = torch.empty(pairs, dtype=torch.int32, device="cuda:0"), torch.empty(pairs, dtype=torch.int32, device="cuda:0")
    row_weight = torch.empty(pairs, device="cuda:0")
    tile_rows = ops.moe_tile_rows(ty, width, inner)
    assert tile_rows == (128 if dtype == "bfloat16" and width % 32 == 0 and inner % 32 == 0 else 16)
    tiles = torch.full((ops.moe_max_tiles(tokens, experts, top, tile_rows), 3), -7, dtype=torch.int32, device="cuda:0")
    ops.moe_route(f32(z), experts, top, 1e-20, chosen, weight, pair_token, place, tiles, tile_rows=tile_rows, router="sigmoid", renormalize=False,
                  row_weight=row_weight)
    up = dev(np.stack([np.concatenate([w[f"e{e}.gate"], w[f"e{e}.up"]]) for e in range(experts)]), ty)
    down = dev(np.stack([w[f"e{e}.down"] for e in range(experts)]), ty)
    got_chosen, wt, pl = chosen.cpu().numpy(), weight.cpu().numpy(), place.cpu().numpy().reshape(tokens, top)
    for t in range(tokens):
        ref_e, ref_w, margin = P.route(z[:, t, :experts].astype(np.float64).sum(0), top)
        if margin > 1e-6 or t == 2:
            assert list(got_chosen[t]) == ref_e and np.allclose(wt[t], ref_w, rtol=1e-5)
    assert np.array_equal(row_weight.cpu().numpy()[pl.reshape(-1)], wt.reshape(-1))
    for weighed in (True, False):
        mid = ops.moe_expert_gated(dev(x, ty), pair_token, row_weight if weighed else None, up, tiles, torch.empty((pairs, inner), dtype=ty, device="cuda:0"),
                                   "silu", tile_rows=tile_rows)
        y = ops.moe_expert(mid, None, down, tiles, torch.empty((pairs, width), device="cuda:0"), tile_rows=tile_rows)
        out = ops.moe_combine(y, place, None, None, torch.empty((tokens, width), device="cuda:0")).cpu().numpy()
        ref = np.zeros((tokens, width))
        for t in range(tokens):
            for j in range(top):
                ref[t] += P.expert(w, f"e{got_chosen[t, j]}.", (float(wt[t, j]) if weighed else 1.0) * x[t:t + 1])[0]
        tol = 1e-5 if dtype == "float32" else 2e-2
        assert np.abs(out - ref).max() <= tol * np.abs(ref).max(), (weighed, np.abs(out - ref).max())


@pytest.mark.parametrize("rows, width", [(1, 64), (8, 96), (5, 100), (40, 2560), (3, 2561), (16, 1000)])
def test_scaled_deltas_ride_on_the_norms(rows, width):
    """x += scale * delta column by column: by itself, in the norm's kernel, and at the end of the product that makes the delta
    (which also prepares the norm), with slabs and at widths that are no multiple of 4."""
    import torch
    from kipp_amd.csrc import ops
    from kipp_amd.parts import build_part
    from kipp_amd.config import RMSNormSpec
    from kipp_amd.runtime import ColumnScaled, Runtime
    rng = np.random.default_rng(width)
    x, scale, weight = rng.normal(size=(rows, width)), rng.normal(size=width), rng.normal(size=width)
    delta = rng.normal(size=(3, rows, width))
    want = x + scale * delta.sum(0)
    normed = P.rms_norm(want, weight, 1e-5)
    assert np.allclose(ops.scale_columns(f32(delta), f32(scale), f32(x), add=True).cpu().numpy(), want, rtol=1e-5, atol=1e-5)
    assert np.allclose(ops.scale_columns(f32(delta), f32(scale), torch.empty((rows, width), device="cuda:0")).cpu().numpy(), scale * delta.sum(0), rtol=1e-5, atol=1e-5)
    for ty, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        xd = f32(x)
        out = ops.rmsnorm_scaled_delta(xd, f32(delta), f32(scale), f32(weight), 1e-5, torch.empty((rows, width), dtype=ty, device="cuda:0"))
        assert np.allclose(xd.cpu().numpy(), want, rtol=1e-5, atol=1e-5) and np.allclose(out.float().cpu().numpy(), normed, rtol=tol, atol=tol)
    rt = Runtime("bfloat16")
    norm = build_part("norm", RMSNormSpec(width, 1e-5), rt)
    norm.load({"weight": f32(weight)})
    h = rounded(rng.normal(size=(rows, 64)), "bfloat16")
    m = rounded(rng.normal(size=(width, 64)) * 0.1, "bfloat16")
    product = rt.linear(dev(h, torch.bfloat16), rt.weight(dev(m, torch.bfloat16)), slabs=True, defer=True)
    xd = f32(x)
    got = rt.rows_of(norm.add_forward(xd, ColumnScaled(rt, product, f32(scale)), torch.bfloat16)).float().cpu().numpy()
    want = x + scale * (h @ m.T)
    assert np.allclose(xd.cpu().numpy(), want, rtol=1e-4, atol=1e-4)
    assert np.allclose(got, P.rms_norm(want, weight, 1e-5), rtol=2e-2, atol=2e-2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads, d, dr, dv, rank, rot_dims, fast", [
    (4, 32, 16, 24, 48, 16, True), (5, 24, 8, 20, 36, 8, False), (2, 16, 12, 48, 20, 8, False), (16, 64, 32, 64, 224, 32, True), (3, 8, 6, 8, 298, 6, False),
    (20, 16, 16, 16, 48, 16, False), (1, 8, 2, 130, 30, 2, True), (2, 12, 0, 16, 32, 0, True)])
def test_latent_kernels_without_a_query_latent_and_with_a_key_that_stands_out(dtype, heads, d, dr, dv, rank, rot_dims, fast):
    """Queries straight from the input product, halves of the rotated part turned with each other, a gate a number: prepare,
    absorb, attention over the cached rows and expand against the plain steps; then one latent made to stand out far back, at a
    page's first and last place, among the first tokens and as the row itself, for a prompt row and for single tokens."""
    import torch
    from kipp_amd.csrc import ops
    from kipp_amd.parts.mixer import paged_attention
    from kipp_amd.runtime import Runtime
    from tests.test_gpu_rerizen import PagedCase, attention_batch
    rt = Runtime(dtype)
    act = rt.act_dtype
    rng = np.random.default_rng(heads * 7 + d)
    T, page, scale, eps, base = 150, 16, 0.11, 1e-5, 777.0
    row, hq = rank + dr, heads * (d + dr)
    freq = f32([base ** (-2.0 * i / rot_dims) for i in range(rot_dims // 2)] or [0.0])
    uk, uv = (rounded(rng.normal(size=(heads * n, rank)) / np.sqrt(rank), dtype) for n in (d, dv))
    norm_w = rounded(1 + 0.1 * rng.normal(size=rank), dtype)
    last = T - 1
    turn = (lambda a: P.rotate(a, np.arange(T), rot_dims, base)) if rot_dims else (lambda a: a)
    for key in (None, 0, 1, 79, 80, last):
        proj = rng.normal(size=(T, hq + row + heads * dv + 3)).astype(np.float32)
        if key is not None:         # one latent along a direction, every other one against it
            v = 2.0 * np.sign(rng.normal(size=rank))
            proj[:, hq:hq + rank] += np.where(np.arange(T)[:, None] == key, v, -v)
        x = proj.astype(np.float64)
        c = P.rms_norm(x[:, hq:hq + rank], norm_w, eps)
        kr = turn(x[:, hq + rank:hq + row].reshape(T, 1, dr)).reshape(T, dr)
        if key is not None:         # every head's last query points along the latent of `key`, far longer than any other score
            for h in range(heads):
                along = uk[h * d:(h + 1) * d] @ c[key]
                proj[last, h * (d + dr):h * (d + dr) + d] = 400.0 * along / max(np.linalg.norm(along), 1e-9)
            x = proj.astype(np.float64)
        q = x[:, :hq].reshape(T, heads, d + dr)
        qr = turn(q[..., d:])
        rows_cache = rounded(np.concatenate([c, kr], axis=1), dtype)
        gate = P.sigmoid(x[:, hq + row:hq + row + heads * dv])
        ref = np.zeros((T, heads, dv))
        for h in range(heads):
            ql = rounded(np.concatenate([q[:, h, :d] @ uk[h * d:(h + 1) * d], qr[:, h]], axis=1), dtype)
            s = np.where(np.tril(np.ones((T, T), dtype=bool)), ql @ rows_cache.T * scale, -np.inf)
            p = np.exp(s - s.max(axis=1, keepdims=True))
            p /= p.sum(axis=1, keepdims=True)
            if key is not None:
                assert p[last, key] > 0.99
            ref[:, h] = (p @ rows_cache[:, :rank]) @ uv[h * dv:(h + 1) * dv].T
        ref = ref.reshape(T, heads * dv) * gate
        for queries in (None, [last, 0, 17]):
            whole, case = PagedCase(T, page, None, seed=3), PagedCase(T, page, queries, seed=3)
            cache = torch.zeros((case.pages, 1, page, row), dtype=act, device="cuda:0")
            slabs = f32(np.stack([proj * 0.25, proj * 0.75])) if key is None else f32(proj)
            ops.latent_prepare(slabs, None, cache, whole.positions, whole.seq_of, whole.table, 0, rank, dr, None, f32(norm_w), eps, freq, rot_dims, 1.0,
                               half=True, kv_at=hq)
            ql = ops.latent_absorb(slabs, dev(uk, act), torch.empty((T, heads * row), dtype=act, device="cuda:0"), whole.positions, freq, rot_dims, 1.0,
                                   heads, d, dr, rank, half=True)
            picked = list(range(T)) if queries is None else queries
            use_fast = fast and dtype == "bfloat16"
            widthv = row if use_fast else rank
            lat = torch.zeros((case.rows, heads * widthv), dtype=act, device="cuda:0")
            paged_attention(rt, attention_batch(case, T, queries), ql[picked].contiguous(), lat, cache, cache, page, case.table, heads, 1, row, widthv, scale,
                            None, use_fast)
            uv_t = dev(uv, act).view(heads, dv, rank).transpose(1, 2).contiguous()
            out = ops.latent_expand(lat, uv_t, torch.empty((case.rows, heads * dv), dtype=act, device="cuda:0"), heads, rank, dv,
                                    gate=slabs[..., picked, :].contiguous(), gate_at=hq + row, gate_each=True)
            want = ref[case.pos]
            err = np.abs(out.float().cpu().numpy() - want).max() / np.abs(want).max()
            assert err < (3e-4 if dtype == "float32" else 3e-2), (dtype, key, queries, err)


# =============================================================================== the engine

@pytest.mark.parametrize("dtype, page", [("float32", 16), ("bfloat16", 16), ("bfloat16", 32), ("float32", 8)])
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("cut", ["whole", "tail", "portions", "mixed"])
def test_cuttings_match_plain(folders, shape, dtype, page, cut):
    """Whole prompts, the last tokens one by one, portions of changing size down to two tokens, and mixed batches in a
    pool that only holds the live requests and has four state slots (pages and slots are used again)."""
    folder = folders[(shape, dtype)]
    vocab = P.load_folder(folder)[0]["vocab"]
    requests = requests_of(vocab)
    if cut == "mixed":
        requests.update({f"s{i}": H.random_tokens(900 + i, n, vocab) for i, n in enumerate(LENGTHS)})
        steps = H.mixed(requests, seed=5)
        engine = engine_of(folder, dtype, page, max_tokens=None, num_pages=H.peak_pages(requests, steps, page), max_requests=4)
    else:
        engine = engine_of(folder, dtype, page)
        steps = {"whole": H.whole, "tail": H.tail_one_by_one, "portions": H.changing_portions}[cut](requests)
    got = H.replay(engine, requests, steps)
    for rid, toks in requests.items():
        close(got[rid], plain_logits(folder, toks), TOL[dtype], f"{shape}/{dtype}/{page}/{cut}/{rid}")
    assert engine.cache.free_pages() == [g.pool.num_pages for g in engine.cache.groups]


@pytest.mark.parametrize("shape", SHAPES)
def test_float32_cuttings_are_bitwise_equal(folders, shape):
    """In float32 every sum runs in an order that the token's own position fixes: how the prompt was cut, what else was
    in the batch and which pages and slots were used change no bit."""
    folder = folders[(shape, "float32")]
    requests = requests_of(P.load_folder(folder)[0]["vocab"], seed=3)
    base = H.replay(engine_of(folder, "float32"), requests, H.whole(requests))
    for maker in (H.tail_one_by_one, H.changing_portions, lambda r: H.mixed(r, seed=11)):
        steps = maker(requests)
        order = list(np.random.default_rng(1).permutation(64))
        got = H.replay(engine_of(folder, "float32", page_order=order, max_requests=5), requests, steps)
        for rid in requests:
            assert np.array_equal(got[rid], base[rid]), f"{shape}/{rid}: bits differ between cuttings"


def one_of_each(vocab=90, width=64):
    return {"architecture": "Bipazen", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "layers": [
        {"type": "rglru", "mixer": {"width": 64, "blocks": 4, "conv": 3}, "mlp": {"kind": "moe", "router": {"experts": 4, "top": 2}, "expert": {"ff": 32}}},
        {"type": "latent_attention", "mixer": {"heads": 2, "dim": 16, "rot_dim": 16, "vdim": 16, "kv_rank": 32, "scale": 0.25, "rot": {"base": 100.0, "dims": 16}},
         "mlp": None},
        {"type": "mamba2", "mixer": {"heads": 2, "vdim": 32, "state": 16, "groups": 1, "conv": 4, "norm_groups": 1}, "mlp": None},
        {"type": "rglru", "mixer": {"width": 64, "blocks": 4, "conv": 3}, "mlp": {"kind": "moe", "router": {"experts": 4, "top": 2}, "expert": {"ff": 32}},
         "weights_of": 0}]}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_and_one_slot_that_is_used_again(tmp_path, dtype):
    """200 tokens, most of them decoded, through one state slot and pages that a second request then takes over (its states and
    its filters' last inputs must start at zero, not where the first left them)."""
    folder = write_model(tmp_path / "one", one_of_each(), 8, dtype)
    tokens = {"r": H.random_tokens(77, 200, 90), "next": H.random_tokens(78, 40, 90)}
    engine = engine_of(folder, dtype, 16, max_tokens=None, num_pages=13, max_requests=1)
    steps = [([("r", 10)], [])] + [([("r", 1)], []) for _ in range(60)] + [([("r", 7)], []), ([("r", 2)], [])] \
        + [([("r", 1)], []) for _ in range(121)]
    steps[-1] = (steps[-1][0], ["r"])
    steps += [([("next", 1)], []), ([("next", 1)], []), ([("next", 31)], [])] + [([("next", 1)], []) for _ in range(7)]
    steps[-1] = (steps[-1][0], ["next"])
    got = H.replay(engine, tokens, steps)
    for rid in tokens:
        close(got[rid], plain_logits(folder, tokens[rid]), TOL[dtype], f"one slot/{dtype}/{rid}")
    if dtype == "bfloat16":
        assert engine.graphs.replays > 100          # the single tokens ran as recorded steps


def test_a_run_with_anothers_weights_keeps_a_state_and_a_cache_of_its_own(tmp_path):
    """The same layer twice against the two layers spelled out with equal tensors: the same bits, and twice the cache."""
    from safetensors.torch import load_file, save_file
    cfg = one_of_each()
    cfg["layers"].append(dict(cfg["layers"][1], weights_of=1))
    folder = write_model(tmp_path / "shared", cfg, 3, "float32")
    spelled = json.loads(json.dumps(cfg))
    tensors = load_file(os.path.join(folder, "model.safetensors"))
    for i, layer in enumerate(spelled["layers"]):
        source = layer.pop("weights_of", None)
        if source is not None:
            tensors.update({f"l{i}." + name.split(".", 1)[1]: t.clone() for name, t in list(tensors.items()) if name.startswith(f"l{source}.")})
    other = tmp_path / "spelled"
    other.mkdir()
    (other / "config.json").write_text(json.dumps(spelled))
    save_file(tensors, str(other / "model.safetensors"))
    requests = {"a": H.random_tokens(1, 50, 90), "b": H.random_tokens(2, 9, 90)}
    one, two = engine_of(folder, "float32"), engine_of(str(other), "float32")
    assert [len(g.runs) for g in one.cache.groups] == [2]
    a, b = (H.replay(e, requests, H.mixed(requests, seed=4)) for e in (one, two))
    for rid in requests:
        assert np.array_equal(a[rid], b[rid])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_other_sizes_and_branches(tmp_path, dtype):
    """Widths that are no multiple of 8 or of 32, one block and as many blocks as channels, one tap and many, one expert, every
    expert chosen, a state of 260 numbers, eighteen heads on one cached row, a latent wider than the matrix-core kernels take,
    no rotated part's leftover, layers of one kind only; prompts of more rows than the few-rows products take."""
    lru = lambda width, blocks, conv: {"width": width, "blocks": blocks, "conv": conv}
    ssd = lambda heads, vdim, state, groups, conv, parts: {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": parts}
    lat = lambda heads, d, dr, dv, rank: {"heads": heads, "dim": d, "rot_dim": dr, "vdim": dv, "kv_rank": rank, "scale": 0.2, "rot": {"base": 300.0, "dims": dr}}
    moe = lambda experts, top, ff: {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    layers = [
        {"type": "rglru", "mixer": lru(50, 1, 1), "mlp": None},
        {"type": "latent_attention", "mixer": lat(18, 8, 4, 8, 28), "mlp": moe(1, 1, 20)},
        {"type": "mamba2", "mixer": ssd(1, 20, 260, 1, 1, 1), "mlp": moe(9, 9, 8)},
        {"type": "rglru", "mixer": lru(21, 21, 6), "mlp": moe(33, 3, 64)},
        {"type": "latent_attention", "mixer": lat(1, 3, 2, 300, 330), "mlp": None},
        {"type": "mamba2", "mixer": ssd(12, 4, 8, 4, 7, 6), "mlp": None},
        {"type": "rglru", "mixer": lru(320, 2, 16), "mlp": moe(2, 1, 100)}]
    for width, chosen in ((100, layers), (72, [layers[0], layers[3], layers[6]]), (64, [layers[1], layers[4]])):
        cfg = {"architecture": "Bipazen", "vocab": 77, "width": width, "norm": {"eps": 1e-6}, "layers": chosen}
        folder = write_model(tmp_path / f"odd{width}", cfg, width, dtype)
        requests = {"long": H.random_tokens(1, 330, 77), "short": H.random_tokens(2, 9, 77)}
        for steps in (H.whole(requests), [([("long", 270)], []), ([("long", 59), ("short", 8)], []), ([("long", 1), ("short", 1)], ["long", "short"])]):
            got = H.replay(engine_of(folder, dtype), requests, steps)
            for rid, toks in requests.items():
                close(got[rid], plain_logits(folder, toks), TOL[dtype] * (4 if dtype == "bfloat16" else 1), f"{width}/{dtype}/{rid}")


def random_configuration(rng):
    """A model of the design with every size, the order of its layers and every constant drawn at random."""
    layers = []
    for i in range(rng.randint(3, 6)):
        if layers and rng.random() < 0.3:
            source = rng.randrange(len(layers))
            if "weights_of" not in layers[source]:
                layers.append(dict(json.loads(json.dumps(layers[source])), weights_of=source))
                continue
        kind = rng.choice(["mamba2", "rglru", "latent_attention"])
        if kind == "mamba2":
            groups = rng.choice([1, 2])
            heads = groups * rng.choice([1, 2, 3])
            mixer = {"heads": heads, "vdim": rng.choice([8, 16, 40]), "state": rng.choice([8, 16, 48, 130]), "groups": groups, "conv": rng.choice([1, 2, 4, 7]),
                     "norm_groups": rng.choice([1, heads])}
        elif kind == "rglru":
            blocks = rng.choice([1, 2, 3, 5])
            mixer = {"width": blocks * rng.choice([8, 20, 32, 72]), "blocks": blocks, "conv": rng.choice([1, 2, 3, 4, 9])}
        else:
            dr = rng.choice([2, 8, 16, 24])
            mixer = {"heads": rng.choice([1, 2, 3, 5]), "dim": rng.choice([8, 16, 40]), "rot_dim": dr, "vdim": rng.choice([8, 24, 64]), "kv_rank": rng.choice([16, 40, 96]),
                     "scale": rng.uniform(0.05, 0.4), "rot": {"base": rng.choice([100.0, 10000.0, 500000.0]), "dims": dr}}
        mlp = None
        if rng.random() < 0.8:
            experts = rng.choice([1, 2, 5, 8])
            mlp = {"kind": "moe", "router": {"experts": experts, "top": rng.randint(1, min(4, experts))}, "expert": {"ff": rng.choice([24, 64, 100])}}
        layers.append({"type": kind, "mixer": mixer, "mlp": mlp})
    return {"architecture": "Bipazen", "vocab": rng.choice([300, 512]), "width": rng.choice([96, 128, 160]), "norm": {"eps": rng.choice([1e-5, 1e-6])},
            "layers": layers}


@pytest.mark.parametrize("seed", range(6))
def test_models_drawn_at_random(tmp_path, seed):
    """Sizes, order of layers and constants drawn at random; whole prompts, portions and mixed batches in float32."""
    cfg = random_configuration(random.Random(seed))
    folder = write_model(tmp_path / "drawn", cfg, seed, "float32")
    requests = {f"r{i}": H.random_tokens(seed * 10 + i, n, cfg["vocab"]) for i, n in enumerate([1, 23, 97, 180])}
    for maker in (H.whole, H.changing_portions, lambda r: H.mixed(r, seed=seed)):
        got = H.replay(engine_of(folder, "float32", max_requests=4), requests, maker(requests))
        for rid, toks in requests.items():
            close(got[rid], plain_logits(folder, toks), 2e-8, f"drawn {seed}/{rid}: {json.dumps(cfg)}")


def test_no_kernel_of_the_slow_class_runs_at_ordinary_sizes(tmp_path):
    """Under bfloat16 a cached row of a multiple of 16 numbers runs on the matrix-core attention, no product goes to the library."""
    folder = write_model(tmp_path / "ordinary", one_of_each(), 4, "bfloat16")
    requests = {"a": H.random_tokens(1, 150, 90), "b": H.random_tokens(2, 37, 90)}
    for steps in (H.whole(requests), H.changing_portions(requests), H.tail_one_by_one(requests, tail=40)):
        engine = engine_of(folder, "bfloat16")
        got = H.replay(engine, requests, steps)
        for rid, toks in requests.items():
            close(got[rid], plain_logits(folder, toks), TOL["bfloat16"], f"ordinary/{rid}")
        assert engine.rt.generic_attention_launches == 0 and engine.rt.library_products == 0


def test_recorded_steps_of_a_changing_batch(tmp_path):
    """Three requests decode together from recorded steps while the states go on in their slots and the filters' rings turn;
    one ends early and the batch goes on at another size."""
    folder = write_model(tmp_path / "recorded", one_of_each(), 5, "bfloat16")
    requests = {"a": H.random_tokens(1, 90, 90), "b": H.random_tokens(2, 120, 90), "c": H.random_tokens(3, 75, 90)}
    steps = [([("a", 30), ("b", 51), ("c", 2)], [])]
    fed = {"a": 30, "b": 51, "c": 2}
    while any(fed[r] < len(requests[r]) for r in fed):
        live = [r for r in fed if fed[r] < len(requests[r])]
        for r in live:
            fed[r] += 1
        steps.append(([(r, 1) for r in live], [r for r in live if fed[r] == len(requests[r])]))
    engine = engine_of(folder, "bfloat16")
    got = H.replay(engine, requests, steps)
    for rid, toks in requests.items():
        close(got[rid], plain_logits(folder, toks), TOL["bfloat16"], f"recorded/{rid}")
    assert engine.graphs.replays > 50


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_scheduler(folders, dtype):
    """`generate` (scheduler, continuous batching, tokens chosen on the device) against the plain implementation:
    every generated token is the plain argmax of its position, or within rounding of it."""
    from kipp_amd import generate
    folder = folders[("bipazen-tiny-b", dtype)]
    cfg, w = P.load_folder(folder)
    prompts = [H.random_tokens(5, 3, cfg["vocab"]), H.random_tokens(6, 40, cfg["vocab"]), H.random_tokens(7, 21, cfg["vocab"])]
    outputs = generate(folder, prompts, max_new_tokens=30, dtype=dtype, page_size=16, prefill_chunk=16, max_step_tokens=24)
    margin = 1e-4 if dtype == "float32" else 0.08
    for prompt, out in zip(prompts, outputs):
        assert len(out) == 30
        logits = P.forward_whole(cfg, w, prompt + out)
        for i, tok in enumerate(out):
            row = logits[len(prompt) - 1 + i]
            assert row[tok] >= row.max() - margin * (row.max() - row.min()), (dtype, i)


def test_trace_replay_and_command_line(folders, tmp_path):
    folder = folders[("bipazen-tiny-a", "bfloat16")]
    vocab = P.load_folder(folder)[0]["vocab"]
    toks = H.random_tokens(4, 60, vocab)
    lines = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:33], "want": [0, 32]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[33:35], "want": []}, {"id": "y", "tokens": toks[:7], "want": [6]}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": toks[35:36], "want": [0]}], "end": ["x"]}]
    out = tmp_path / "out"
    run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "bfloat16", "--out", str(out),
                          "--max-tokens", "128"], input="\n".join(json.dumps(l) for l in lines) + "\n", capture_output=True, text=True, timeout=600)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [l for l in run.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    ref = plain_logits(folder, toks)
    for step, places in ((0, [0, 32]), (1, [6]), (2, [35])):
        rows = np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(len(places), vocab)
        each = np.sum((rows - ref[places]) ** 2, axis=1) / np.sum(ref[places] ** 2, axis=1)
        margins = np.minimum.accumulate(_margin_cache[id(ref)])[places]
        assert np.all((each <= TOL["bfloat16"]) | (margins < CLOSE_CALL)), (step, each)
    cli = subprocess.run([sys.executable, "-m", "kipp_amd.cli", "--model", folder, "--tokens", ",".join(map(str, toks[:9])), "--decode", "5"],
                         capture_output=True, text=True, timeout=600, cwd=ROOT)
    assert cli.returncode == 0, cli.stderr[-2000:]
