"""The Bavedra design on the GPU against its plain implementation: every new kernel alone (crafted inputs at the edges), then
the engine under every cutting in both precisions, tight pools, slots used again, long decoding, recorded steps, other sizes,
models drawn at random, generation through the scheduler, the trace replay and the command line.  (The kernels of the delta
rule, the state space layer and the recurrence are shared with other designs, whose tests run them alone.)"""
import json
import os
import random
import subprocess
import sys

import numpy as np
import pytest

from tests import helpers as H
from tests.plain import bavedra_plain as P

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
SHAPES = ("bavedra-tiny-a", "bavedra-tiny-b")
LENGTHS = [1, 19, 45, 80, 131]
TOL = {"float32": 1e-9, "bfloat16": 2e-2}     # float32 is the sharp test


def sharpen(folder):
    """Larger query, key and router matrices, so that few keys carry a row's softmax and experts are told apart; decays near one,
    so that a lost state shows far behind."""
    from safetensors import safe_open
    from safetensors.torch import save_file
    path = os.path.join(folder, "model.safetensors")
    with safe_open(path, framework="pt") as f:
        tensors = {name: f.get_tensor(name) for name in f.keys()}
    for name, t in tensors.items():
        if name.endswith((".left.q", ".left.k", ".mlp.router", ".shared.sg")):
            tensors[name] = (t.float() * 8.0).to(t.dtype)
        elif name.endswith(".mix.lam"):
            tensors[name] = (t.float() - 5.0).to(t.dtype)
        elif name.endswith(".A_log"):
            tensors[name] = (t.float() - 3.0).to(t.dtype)
    save_file(tensors, path)
    return folder


def write_model(path, cfg, seed, dtype):
    from kipp_amd.weights import write_random_model
    return sharpen(write_random_model(str(path), cfg, seed=seed, dtype=dtype))


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    from kipp_amd.config import shape_config
    root = tmp_path_factory.mktemp("bavedra")
    return {(shape, dtype): write_model(root / f"{shape}-{dtype}", shape_config(shape), 70 + i, dtype)
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
CLOSE_CALL = 0.01   # a router's margin (in scores of a softmax) below which bfloat16 rows may choose another expert


def close(got, ref, tol, what):
    """Every position's normalised squared error within `tol`.  Under the bfloat16 bound a router's choice between two experts
    whose scores differ by less than the rounding of the rows it reads falls either way, and the position (and, through the
    states and keys, every one after it) then differs by much more than rounding: a request passes if every position beyond
    the bound stands at or behind a close call of the plain implementation's routers, or if no more than a share of its
    positions lie beyond it.  The float32 runs of the same cases, and models without a router, allow no such position."""
    assert got.shape == ref.shape and np.isfinite(got).all(), what
    each = [float(np.sum((g - r) ** 2) / np.sum(r ** 2)) for g, r in zip(got.astype(np.float64), ref)]
    margins = _margin_cache.get(id(ref)) if tol >= TOL["bfloat16"] else None
    spared = 0
    if margins is not None:
        spared = int(FLIPS * len(each))
        called = np.minimum.accumulate(margins[:len(each)]) < CLOSE_CALL
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


# =============================================================================== the kernels alone

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H_, G, d, rot, window, page, fast", [(4, 2, 32, 16, 40, 16, True), (6, 2, 24, 24, 11, 8, False), (3, 3, 97, 2, 17, 16, False),
                                                              (2, 1, 200, 64, 64, 32, False), (2, 2, 64, 64, 1, 16, True), (8, 2, 128, 128, 150, 16, True),
                                                              (4, 1, 16, 6, 33, 8, True), (2, 2, 256, 100, 16, 16, False)])
def test_keys_that_are_the_values_and_a_key_that_stands_out(dtype, H_, G, d, rot, window, page, fast):
    """Heads made ready (neighbours turned, the unturned key as the value, from slabs, with and without a bias) and the windowed
    attention with the added one, on the generic kernel and, where the sizes allow it under bfloat16, on the matrix cores: random
    inputs; then one key whose score stands out, far below zero everywhere else, at the window's edge, just outside, at page
    borders, first of all and the row itself: the last row of a prompt portion and a single token give that key when the window
    holds it and (the added one carrying the row) nothing when it does not."""
    import torch
    from kipp_amd.csrc import ops
    from kipp_amd.parts.mixer import paged_attention
    from kipp_amd.runtime import Runtime
    from tests.test_gpu_rerizen import PagedCase, attention_batch
    rt = Runtime(dtype)
    act = rt.act_dtype
    rng = np.random.default_rng(d + window)
    T, scale, base = 150, 0.3, 700.0
    freq = f32([base ** (-2.0 * i / rot) for i in range(rot // 2)])
    last = T - 1

    def run(proj, queries, bias=None, split=False):
        whole, case = PagedCase(T, page, None, seed=3), PagedCase(T, page, queries, seed=3)
        kc, vc = (torch.zeros((case.pages, G, page, d), dtype=act, device="cuda:0") for _ in range(2))
        angles = ops.rotary_angles(whole.positions, freq, torch.empty((T, rot), device="cuda:0"))
        pd = f32(np.stack([0.25 * proj, 0.75 * proj])) if split else f32(proj)
        q = ops.head_prepare(pd, torch.empty((T, H_ * d), dtype=act, device="cuda:0"), kc, vc, whole.positions, whole.seq_of, whole.table, H_, G, d, d,
                             None if bias is None else f32(bias), "none", 0.0, angles=angles, rotary_dim=rot, interleaved=True, keys_as_values=True)
        picked = list(range(T)) if queries is None else queries
        outs = []
        for use_fast in ([False, True] if fast and dtype == "bfloat16" else [False]):
            out = torch.zeros((case.rows, H_ * d), dtype=act, device="cuda:0")
            paged_attention(rt, attention_batch(case, T, queries), q[picked].contiguous(), out, kc, vc, page, case.table, H_, G, d, d, scale, window, use_fast, sink=True)
            outs.append(out.float().cpu().numpy().reshape(case.rows, H_, d))
        return outs, case

    proj = rng.normal(size=(T, (H_ + G) * d + 3)).astype(np.float32)
    bias = rng.normal(size=(H_ + G) * d).astype(np.float32) * 0.3
    tol = 2e-4 if dtype == "float32" else 4e-2
    for b in (None, bias):
        p64 = proj[:, :(H_ + G) * d].astype(np.float64) + (0.0 if b is None else b)
        q, k = p64[:, :H_ * d].reshape(T, H_, d), p64[:, H_ * d:].reshape(T, G, d)
        ref = P.window_attention_core(P.rotate_neighbours(q, range(T), rot, base), P.rotate_neighbours(k, range(T), rot, base), k, scale, window)
        for queries in (None, [last, 0, 17]):
            outs, case = run(proj, queries, b, split=b is not None)
            for out in outs:
                assert np.allclose(out, ref[case.pos], rtol=tol, atol=tol), (queries, np.abs(out - ref[case.pos]).max())
    # every turned key lies along one direction (the one of `key` turned there), `key` with it and all others against it
    u = rng.normal(size=d)
    u *= 20.0 / np.linalg.norm(u)
    edge = last - window + 1
    for key in sorted({edge, edge - 1, edge + 1, 0, 1, last, last - 1, last // page * page, last // page * page - 1, T // 2} & set(range(T))):
        along = P.rotate_neighbours(u.reshape(1, 1, d), [key], rot, base)[0, 0]
        rows = np.stack([P.rotate_neighbours(along.reshape(1, 1, d), [-t], rot, base)[0, 0] for t in range(T)])
        crafted = np.zeros_like(proj)
        crafted[:, H_ * d:(H_ + G) * d] = np.tile(np.where(np.arange(T)[:, None] == key, rows, -rows), (1, G))
        crafted[last, :H_ * d] = np.tile(rows[last], H_)
        seen = last - key < window
        want = u if seen else np.zeros(d)
        for queries in (None, [last]):
            for out in run(crafted, queries)[0]:
                assert np.allclose(out[-1], np.tile(want, (H_, 1)), atol=0.15), (key, seen, queries, np.abs(out[-1] - want).max())


@pytest.mark.parametrize("n_q, n_kv, d, page, window, build", [
    (4, 2, 32, 16, 40, None), (8, 2, 128, 16, 100, None), (3, 3, 64, 8, 7, None), (8, 2, 128, 16, 1024, None), (8, 2, 128, 16, 1500, "STREAM_FROM"),
    (8, 2, 128, 16, 300, "RING_FROM_PAIRS"), (8, 2, 128, 16, 4096, "RING_FROM_PAIRS"), (4, 1, 16, 32, 64, None), (4, 1, 16, 16, 1, None)])
def test_windows_with_the_added_one_on_the_matrix_cores(n_q, n_kv, d, page, window, build):
    """The builds of the matrix-core attention that add one to the denominator, with a window, for prompt portions and for single
    tokens (also the kernels for long contexts and for whole contexts, built so that small inputs reach them), against the sum
    written out here: sequence lengths just past, at and just before the window's length; scores of every size, so that the
    added one is anything from all of a row's denominator to nothing of it."""
    import torch
    from kipp_amd.csrc import ops
    rng = np.random.default_rng(n_q + d + window + len(build or ""))
    scale = 1.7 / np.sqrt(d)
    seq_lens = [1, 70, 300, 257, 129, window + 1, window, 2 * window + 1][:5 if window > 600 else 8] + ([2300, 1025] if build else [])
    q_lens = [1, 70, 130, 2, 129, 2, min(window, 60), 3][:5 if window > 600 else 8] + ([200, 1] if build else [])
    q_lens = [min(a, b) for a, b in zip(q_lens, seq_lens)]
    blocks = [-(-n // page) for n in seq_lens]
    perm = rng.permutation(sum(blocks) + 3)
    table = np.zeros((len(seq_lens), max(blocks)), dtype=np.int32)
    at = 0
    for i, b in enumerate(blocks):
        table[i, :b] = perm[at:at + b]
        at += b
    k = torch.tensor(rng.normal(size=(len(perm), n_kv, page, d)), dtype=torch.bfloat16)
    v = torch.tensor(rng.normal(size=(len(perm), n_kv, page, d)) + 1.0, dtype=torch.bfloat16)

    def keys_of(cache, seq, lo, n):
        return np.stack([cache[table[seq, j // page], :, j % page, :].double().numpy() for j in range(lo, n)])

    def expected(qrow, seq, pos):
        lo = max(0, pos - window + 1)
        ks, vs = keys_of(k, seq, lo, pos + 1), keys_of(v, seq, lo, pos + 1)
        out = np.zeros((n_q, d))
        for h in range(n_q):
            g = h // (n_q // n_kv)
            sc = (ks[:, g] @ qrow[h]) * scale
            top = max(sc.max(), 0.0)
            w = np.exp(sc - top)
            out[h] = (w / (w.sum() + np.exp(-top))) @ vs[:, g]
        return out

    def queries(rows):
        """Random ones, a third of them short: their scores are near zero."""
        q = rng.normal(size=(rows, n_q, d))
        q[::3] *= 0.01
        return torch.tensor(q.reshape(rows, n_q * d), dtype=torch.bfloat16)

    inner = ops._fn
    if build:
        ops._fn = lambda lib, name, argtypes, defines=None: inner(lib, name, argtypes, dict(defines, **{build: 1024 if build == "STREAM_FROM" else 1}) if lib == "attention_decode" else defines)
    try:
        positions, seq_of, q_start = [], [], []
        for i, (n, ql) in enumerate(zip(seq_lens, q_lens)):
            q_start.append(len(positions))
            positions += list(range(n - ql, n))
            seq_of += [i] * ql
        t = len(positions)
        q = queries(t)
        items = [(i, tile) for i, ql in enumerate(q_lens) for tile in range(-(-ql // 128))]
        out = ops.attention_prefill(q.cuda(), k.cuda(), v.cuda(), torch.zeros(t, n_q * d, dtype=torch.bfloat16, device="cuda:0"),
                                    i32([i for i, _ in items]), i32([tile for _, tile in items]), i32(q_start), i32(q_lens), i32(positions),
                                    i32(table), n_q, n_kv, d, scale, window, sink=True).float().cpu().numpy().reshape(t, n_q, d)
        qd = q.double().numpy().reshape(t, n_q, d)
        for row in sorted(set(list(range(0, t, 17)) + q_start + [s + ql - 1 for s, ql in zip(q_start, q_lens)])):
            ref = expected(qd[row], seq_of[row], positions[row])
            assert np.abs(out[row] - ref).max() < 2e-2 * max(1.0, np.abs(ref).max()), ("portion", row, seq_of[row], positions[row])
        n_seq = len(seq_lens)
        rows = list(range(2, n_seq + 2))
        pos1, seq1 = [0, 0] + [n - 1 for n in seq_lens], [0, 0] + list(range(n_seq))
        q1 = queries(n_seq + 2)
        out1 = torch.zeros(n_seq + 2, n_q * d, dtype=torch.bfloat16, device="cuda:0")
        ws = ops.attention_decode_workspace(n_seq, n_q, d, max(seq_lens), "cuda:0")
        ops.attention_decode(q1.cuda(), k.cuda(), v.cuda(), out1, i32(rows), i32(pos1), i32(seq1), i32(table), n_q, n_kv, d, scale, window,
                             max(seq_lens), ws, sink=True)
        got = out1.float().cpu().numpy().reshape(n_seq + 2, n_q, d)
        q1d = q1.double().numpy().reshape(n_seq + 2, n_q, d)
        for r in rows:
            ref = expected(q1d[r], seq1[r], pos1[r])
            assert np.abs(got[r] - ref).max() < 2e-2 * max(1.0, np.abs(ref).max()), ("single token", r, pos1[r])
        assert not got[:2].any()
    finally:
        ops._fn = inner


@pytest.mark.parametrize("rows, width", [(1, 64), (8, 96), (5, 101), (300, 320), (3, 2561), (40, 2560), (260, 2560), (9, 4096), (2, 8192), (300, 3000), (257, 8000), (1, 9001)])
def test_normed_results_are_added_and_normed_again_in_one_kernel(rows, width):
    """x += sum of scale * N(delta) and the next norm of it, for one and two terms of very different sizes (one so small that its
    eps counts), in slabs, with and without the next norm; by the norm part that a block calls, and as a tensor of its own."""
    import torch
    from kipp_amd.config import RMSNormSpec
    from kipp_amd.csrc import ops
    from kipp_amd.parts import build_part
    from kipp_amd.parts.norm import NormedSum
    from kipp_amd.runtime import Runtime
    rng = np.random.default_rng(width + rows)
    x = rng.normal(size=(rows, width))
    deltas = [np.float32(rng.normal(size=(5, rows, width)) * 40.0), np.float32(rng.normal(size=(1, rows, width)) * 2e-3)]
    weights, scales, eps = [rng.normal(size=width) for _ in range(2)], (0.5, -1.25), (1e-5, 3e-6)
    nw = rng.normal(size=width)
    part = [s * P.rms_norm(d.astype(np.float64).sum(0), np.float32(w), e) for d, w, s, e in zip(deltas, weights, scales, eps)]
    for terms in ((0, 1), (1,), (0,), (1, 0)):
        want = np.float32(x).astype(np.float64) + sum(part[k] for k in terms)
        given = [(f32(deltas[k] if k == 0 else deltas[k][0]), f32(weights[k]), eps[k], scales[k]) for k in terms]
        for ty, tol in ((torch.float32, 2e-5), (torch.bfloat16, 1e-2)):
            xd = f32(x)
            out = torch.empty((rows, width), dtype=ty, device="cuda:0")
            ops.normed_sum_step(xd, given, f32(nw), 1e-6, out)
            assert np.allclose(xd.cpu().numpy(), want, rtol=2e-5, atol=2e-5)
            assert np.allclose(out.float().cpu().numpy(), P.rms_norm(want, np.float32(nw), 1e-6), rtol=tol, atol=tol * 3)
        xd = f32(x)
        ops.normed_sum_step(xd, given)
        assert np.allclose(xd.cpu().numpy(), want, rtol=2e-5, atol=2e-5)
    rt = Runtime("bfloat16")
    norms = [build_part("norm", RMSNormSpec(width, e), rt) for e in eps + (1e-6,)]
    for norm, w in zip(norms, weights + [nw]):
        norm.load({"weight": f32(w)})
    pending = NormedSum(rt, [(f32(deltas[0]), norms[0], scales[0]), (f32(deltas[1]), norms[1], scales[1])])
    assert np.allclose(rt.settle(pending).cpu().numpy(), part[0] + part[1], rtol=2e-5, atol=2e-5)
    xd = f32(x)
    got = norms[2].add_forward(xd, pending, torch.float32)
    assert np.allclose(got.cpu().numpy(), P.rms_norm(np.float32(x) + part[0] + part[1], np.float32(nw), 1e-6), rtol=2e-5, atol=1e-4)


@pytest.mark.parametrize("k, n", [(64, 96), (72, 50), (320, 256), (2560, 1000), (96, 33), (512, 2048)])
def test_products_that_end_in_the_square_of_relu(k, n):
    """For few rows (from rows and from tiles, with a row scale left by a norm, in and out of steps-major order), for a few dozen
    and for hundreds (the planned cut and forced ones): against the product and the activation in float64."""
    import torch
    from kipp_amd.csrc import ops
    rng = np.random.default_rng(k + n)
    w = rounded(rng.normal(size=(n, k)) / np.sqrt(k), "bfloat16")
    wd = dev(w, torch.bfloat16)
    tiles = ops.tile_weight(wd) if k % 32 == 0 else None

    def check(out, ref, what):
        assert np.allclose(out.float().cpu().numpy(), ref, rtol=1e-2, atol=2e-3), (what, np.abs(out.float().cpu().numpy() - ref).max())
    for m in (1, 7, 16, 17, 40, 64):
        x = rounded(rng.normal(size=(m, k)) * 2, "bfloat16")
        xd = dev(x, torch.bfloat16)
        ref = np.maximum(x @ w.T, 0.0) ** 2
        empty = lambda: torch.full((m, n), 7.0, dtype=torch.bfloat16, device="cuda:0")
        for t in (None, tiles):
            check(ops.gemm_skinny_relu2(xd, wd, empty(), tiles=t), ref, ("few", m, t is None))
            check(ops.gemm_rows_relu2(xd, wd, empty(), tiles=t), ref, ("dozens", m, t is None))
        if m <= 16:
            parts = 3
            sums = rng.uniform(0.5, 2.0, size=(m, 4)).astype(np.float32)
            sums[:, 3] = 100.0          # beyond the parts: not read
            scaled = x / np.sqrt(sums[:, :3].sum(1, keepdims=True) / k + 1e-5)
            out = ops.gemm_skinny_relu2(xd, wd, empty(), tiles=tiles, row_scale=(f32(sums), parts, 1e-5))
            assert np.allclose(out.float().cpu().numpy(), np.maximum(scaled @ w.T, 0) ** 2, rtol=2e-2, atol=1e-2 * np.maximum(scaled @ w.T, 0).max() ** 2)
            if k % 32 == 0:
                check(ops.gemm_skinny_relu2(ops.steps_major(xd), wd, empty(), tiles=tiles, x_steps_major=True), ref, "x in steps")
                if n % 32 == 0:
                    check(ops.from_steps_major(ops.gemm_skinny_relu2(xd, wd, empty(), tiles=tiles, out_steps_major=True)), ref, "out in steps")
    if k % 32 == 0:
        for m in (65, 200, 300):
            x = rounded(rng.normal(size=(m, k)) * 2, "bfloat16")
            ref = np.maximum(x @ w.T, 0.0) ** 2
            xd = dev(x, torch.bfloat16)
            check(ops.gemm_tiles(xd, wd, end="relu2"), ref, ("many", m))
            for cut in (441, 421, 241, 1421, 2421):
                check(ops.gemm_tiles(xd, wd, end="relu2", force=cut), ref, ("many", m, cut))
            if m <= 256:
                check(ops.gemm_rows_relu2(xd, wd, torch.empty((m, n), dtype=torch.bfloat16, device="cuda:0"), tiles=tiles), ref, ("dozens", m))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("activation", ["relu2", "silu", "gelu_tanh"])
@pytest.mark.parametrize("width, inner", [(64, 96), (100, 52), (320, 1024)])
def test_the_feed_forward_without_a_gate(dtype, activation, width, inner):
    import torch
    from kipp_amd.config import DenseMLPSpec
    from kipp_amd.parts import build_part
    from kipp_amd.runtime import Runtime
    rt = Runtime(dtype)
    rng = np.random.default_rng(width + inner)
    w = {"up": rounded(rng.normal(size=(inner, width)) / np.sqrt(width), dtype), "down": rounded(rng.normal(size=(width, inner)) / np.sqrt(inner), dtype)}
    part = build_part("feed_forward", DenseMLPSpec(width, inner, activation), rt)
    part.load({name: dev(t, rt.act_dtype) for name, t in w.items()})
    act = {"relu2": lambda z: np.maximum(z, 0) ** 2, "silu": P.silu, "gelu_tanh": P.gelu_tanh}[activation]
    for rows in (1, 5, 12, 13, 40, 100, 300):
        x = rounded(rng.normal(size=(rows, width)), dtype)
        y = rt.settle(part.forward(dev(x, rt.act_dtype)))
        y = (y.sum(0) if y.dim() == 3 else y).cpu().numpy()
        ref = act(x @ w["up"].T) @ w["down"].T
        assert np.abs(y - ref).max() < (1e-4 if dtype == "float32" else 2e-2) * np.abs(ref).max(), (rows, np.abs(y - ref).max())


@pytest.mark.parametrize("experts, identity, top, count, keep, tokens", [(16, 4, 2, 4, 2, 37), (10, 5, 3, 5, 2, 300), (6, 0, 3, 3, 2, 1), (5, 3, 2, 1, 1, 20),
                                                                        (60, 12, 8, 9, 4, 129), (2, 7, 4, 3, 2, 40), (130, 2, 4, 66, 3, 40), (1, 1, 2, 1, 1, 5)])
def test_softmax_router_with_correction_groups_and_identity_experts(experts, identity, top, count, keep, tokens):
    """The correction in the choice but not in the weights, negative choice scores, groups by their largest, exact ties; identity
    experts among the choices have no row: the other pairs are sorted into runs of one expert, each covered by one tile."""
    import torch
    from kipp_amd.csrc import ops
    rng = np.random.default_rng(experts * 7 + top)
    e_all, pairs = experts + identity, tokens * top
    z = rng.normal(size=(2, tokens, e_all + 3)).astype(np.float32) * 2
    for corr in (rng.normal(size=e_all).astype(np.float32) * (1.0 / e_all), rng.normal(size=e_all).astype(np.float32) * 0.01 - 2.0):
        corr[e_all // 2] += 1.0
        if tokens > 3:
            z[:, 3, :e_all] = 0.125         # every score equal: the correction and then the index decide
            corr[1:e_all // 2] = corr[0]
        chosen, weight = torch.empty((tokens, top), dtype=torch.int32, device="cuda:0"), torch.empty((tokens, top), device="cuda:0")
        pair_token, place = torch.empty(pairs, dtype=torch.int32, device="cuda:0"), torch.empty(pairs, dtype=torch.int32, device="cuda:0")
        tiles = torch.full((ops.moe_max_tiles(tokens, experts, top), 3), -7, dtype=torch.int32, device="cuda:0")
        ops.moe_route(f32(z), experts, top, 1e-20, chosen, weight, pair_token, place, tiles, correction=f32(corr), groups=(count, keep), identity=identity,
                      group_score="top1")
        got, wt, pl, pt, tl = (t.cpu().numpy() for t in (chosen, weight, place.view(tokens, top), pair_token, tiles))
        for t in range(tokens):
            ref_e, ref_w, margin = P.route(z[:, t, :e_all].astype(np.float64).sum(0), corr.astype(np.float64), top, count, keep)
            assert len(set(got[t])) == top and np.isclose(wt[t].sum(), 1.0, rtol=1e-5)
            if margin > 1e-6 or (t == 3 and margin == 0.0):
                assert list(got[t]) == ref_e and np.allclose(wt[t], ref_w, rtol=1e-5, atol=1e-9), (t, got[t], ref_e, wt[t], ref_w)
        real = got < experts
        assert np.all(pl[~real] == -1) and sorted(pl[real].tolist()) == list(range(int(real.sum())))
        expert_of_row = np.empty(int(real.sum()), dtype=np.int64)
        expert_of_row[pl[real]] = got[real]
        assert np.all(np.diff(expert_of_row) >= 0) and np.array_equal(pt[pl[real]], np.nonzero(real)[0])
        covered = np.zeros(len(expert_of_row), dtype=int)
        for ex, first, rows in tl:
            assert 0 <= rows <= 16
            if rows:
                assert np.all(expert_of_row[first:first + rows] == ex)
                covered[first:first + rows] += 1
        assert np.all(covered == 1)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("experts, identity, top, count, keep, width, inner, shared", [
    (8, 4, 3, 4, 2, 64, 96, 160), (5, 1, 2, 2, 1, 40, 30, 20), (3, 5, 4, 1, 1, 101, 24, 0), (6, 0, 2, 3, 2, 96, 64, 96), (16, 16, 4, 8, 4, 320, 128, 256)])
def test_routed_feed_forward_with_identity_experts_and_a_weighed_shared_one(dtype, experts, identity, top, count, keep, width, inner, shared):
    """The whole part for 1 to 300 rows against loops over tokens (rows whose choice is a close call under bfloat16 are left out)."""
    import torch
    from kipp_amd.config import RoutedMLPSpec
    from kipp_amd.parts import build_part
    from kipp_amd.runtime import Runtime
    rt = Runtime(dtype)
    rng = np.random.default_rng(experts + width)
    spec = RoutedMLPSpec(hidden_size=width, experts=experts, top=top, expert_size=inner, shared_size=shared or None, activation="silu", correction_name="correction",
                         groups=(count, keep), group_score="top1", gate_name="gate", identity=identity, shared_gate_name="shared.sg" if shared else None)
    part = build_part("feed_forward", spec, rt)
    w = {}
    for name, p in part.params(spec).items():
        a = rng.normal(size=p.shape) * (0.5 / spec.choices if name == "correction" else 2.0 / np.sqrt(width))
        w[name] = a.astype(np.float32).astype(np.float64) if name == "correction" else rounded(a, dtype)
    part.load({name: dev(t, torch.float32 if name == "correction" else rt.act_dtype) for name, t in w.items()})
    mlp = {"router": {"experts": experts, "identity": identity, "top": top, "groups": {"count": count, "keep": keep}}, "shared": {"ff": shared} if shared else None}
    for rows in (1, 6, 30, 300):
        x = rounded(rng.normal(size=(rows, width)), dtype)
        out = part.forward(dev(x, rt.act_dtype)).cpu().numpy()
        margins = []
        ref = P.routed_ff(w, "", mlp, x, margins)
        clear = np.array(margins) > 1e-4
        tol = 1e-4 if dtype == "float32" else 3e-2
        assert clear.sum() > 0.8 * rows - 1
        assert np.abs(out - ref)[clear].max() < tol * np.abs(ref).max(), (rows, np.abs(out - ref)[clear].max(), np.abs(ref).max())


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


def moe(experts, identity, top, count, keep, ff, shared=None):
    return {"kind": "moe", "router": {"experts": experts, "identity": identity, "top": top, "groups": {"count": count, "keep": keep}}, "expert": {"ff": ff},
            "shared": {"ff": shared} if shared else None}


def side_by_side(heads, kv, d, window, rot, s_heads, vdim, state, groups, conv, parts, base=500.0, scale=0.2):
    return {"left": {"heads": heads, "kv_heads": kv, "dim": d, "vdim": d, "mask": {"size": window}, "rot": {"base": base, "dims": rot}, "scale": scale},
            "right": {"heads": s_heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": parts}}


def model_of(layers, vocab=90, width=64, scale=5.0, eps=1e-5):
    return {"architecture": "Bavedra", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps}, "layers": layers}


def one_of_each():
    return model_of([
        {"type": "parallel", "mixer": side_by_side(2, 1, 16, 30, 8, 2, 32, 16, 1, 4, 2), "mlp": moe(4, 2, 2, 2, 1, 32, 64)},
        {"type": "delta", "mixer": {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 16, "conv": 3}, "mlp": {"kind": "dense", "ff": 128}},
        {"type": "rglru", "mixer": {"width": 64, "blocks": 4, "conv": 3}, "mlp": None},
        {"type": "parallel", "mixer": side_by_side(2, 1, 16, 30, 8, 2, 32, 16, 1, 4, 2), "mlp": moe(4, 2, 2, 2, 1, 32, 64), "weights_of": 0}])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["parallel", "delta", "rglru", "dense", "moe"])
def test_each_mechanism_alone_in_a_model(tmp_path, kind, dtype):
    """Two layers of one mechanism: a prompt whole, then token by token from the first, then in portions."""
    layers = one_of_each()["layers"]
    layer = {"parallel": dict(layers[0], mlp=None), "delta": dict(layers[1], mlp=None), "rglru": layers[2], "dense": dict(layers[2], mlp=layers[1]["mlp"]),
             "moe": dict(layers[2], mlp=layers[0]["mlp"])}[kind]
    folder = write_model(tmp_path / kind, model_of([layer, json.loads(json.dumps(layer))]), 21, dtype)
    requests = {"a": H.random_tokens(31, 70, 90), "b": H.random_tokens(32, 37, 90)}
    for steps in (H.whole(requests), H.tail_one_by_one(requests, tail=69), H.changing_portions(requests)):
        got = H.replay(engine_of(folder, dtype), requests, steps)
        for rid, toks in requests.items():
            close(got[rid], plain_logits(folder, toks), TOL[dtype], f"{kind}/{dtype}/{rid}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_and_one_slot_that_is_used_again(tmp_path, dtype):
    """200 tokens, most of them decoded, through one state slot and few pages that a second request then takes over (its states
    and its filters' last inputs must start at zero, not where the first left them; the window's pages went back long ago)."""
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
    """The same layers twice against layers spelled out with equal tensors: the same bits, and twice the cache."""
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
    """Widths that are no multiple of 8 or of 32, heads of 3 and of 256 numbers, a head turned whole and by one pair, windows of
    one and longer than the prompt, twenty query heads on one key, one tap and many, one expert, all chosen, none but identity
    experts kept, a state of 260 numbers, layers of one kind only; prompts of more rows than the few-rows products take."""
    delta = lambda heads, kv, d, dv, conv: {"heads": heads, "kv_heads": kv, "dim": d, "vdim": dv, "conv": conv}
    lru = lambda width, blocks, conv: {"width": width, "blocks": blocks, "conv": conv}
    dense = lambda ff: {"kind": "dense", "ff": ff}
    layers = [
        {"type": "parallel", "mixer": side_by_side(20, 1, 8, 50, 8, 1, 20, 260, 1, 1, 1), "mlp": moe(1, 1, 1, 2, 1, 20)},
        {"type": "delta", "mixer": delta(5, 1, 7, 9, 1), "mlp": dense(35)},
        {"type": "parallel", "mixer": side_by_side(3, 3, 3, 1, 2, 12, 4, 8, 4, 7, 6), "mlp": moe(9, 0, 9, 1, 1, 8, 5)},
        {"type": "rglru", "mixer": lru(50, 1, 1), "mlp": moe(2, 6, 3, 4, 2, 64, 100)},
        {"type": "parallel", "mixer": side_by_side(2, 1, 256, 1000, 100, 4, 16, 24, 2, 3, 1), "mlp": None},
        {"type": "delta", "mixer": delta(4, 4, 130, 40, 16), "mlp": moe(33, 7, 3, 5, 3, 64, 32)},
        {"type": "rglru", "mixer": lru(320, 2, 16), "mlp": dense(200)}]
    for width, chosen in ((100, layers), (72, [layers[0], layers[3], layers[6]]), (64, [layers[2], layers[5]]), (31, [layers[1], layers[4]])):
        folder = write_model(tmp_path / f"odd{width}", model_of(chosen, vocab=77, width=width, eps=1e-6), width, dtype)
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
        kind = rng.choice(["parallel", "delta", "rglru"])
        if kind == "parallel":
            kv, groups, d = rng.choice([1, 2, 3]), rng.choice([1, 2]), rng.choice([8, 16, 20, 48, 64])
            s_heads = groups * rng.choice([1, 2, 3])
            mixer = side_by_side(kv * rng.choice([1, 2, 4]), kv, d, rng.choice([1, 5, 16, 37, 90, 400]), 2 * rng.randint(1, d // 2), s_heads, rng.choice([8, 16, 40]),
                                 rng.choice([8, 16, 48, 130]), groups, rng.choice([1, 2, 4, 7]), rng.choice([1, s_heads]), rng.choice([100.0, 10000.0]),
                                 rng.uniform(0.05, 0.4))
        elif kind == "delta":
            kv = rng.choice([1, 2, 3])
            mixer = {"heads": kv * rng.choice([1, 2, 3]), "kv_heads": kv, "dim": rng.choice([8, 20, 32, 70]), "vdim": rng.choice([8, 24, 64]),
                     "conv": rng.choice([1, 2, 4, 6])}
        else:
            blocks = rng.choice([1, 2, 3, 5])
            mixer = {"width": blocks * rng.choice([8, 20, 32, 72]), "blocks": blocks, "conv": rng.choice([1, 2, 3, 4, 9])}
        mlp = None
        if rng.random() < 0.4:
            mlp = {"kind": "dense", "ff": rng.choice([40, 96, 200])}
        elif rng.random() < 0.8:
            count, size = rng.choice([1, 2, 3, 4]), rng.choice([2, 3, 5])
            keep = rng.randint(1, count)
            identity = rng.randint(0, min(5, count * size - 1))
            mlp = moe(count * size - identity, identity, rng.randint(1, min(4, keep * size)), count, keep, rng.choice([24, 64, 100]), rng.choice([None, 48, 96]))
        layers.append({"type": kind, "mixer": mixer, "mlp": mlp})
    return model_of(layers, rng.choice([300, 510]), rng.choice([96, 128, 150]), rng.choice([1.0, 3.5, 11.0]), rng.choice([1e-5, 1e-6]))


@pytest.mark.parametrize("seed", range(8))
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
    """Under bfloat16 heads of a multiple of 16 numbers run on the matrix-core attention, no product goes to the library."""
    folder = write_model(tmp_path / "ordinary", one_of_each(), 4, "bfloat16")
    requests = {"a": H.random_tokens(1, 150, 90), "b": H.random_tokens(2, 37, 90)}
    for steps in (H.whole(requests), H.changing_portions(requests), H.tail_one_by_one(requests, tail=40)):
        engine = engine_of(folder, "bfloat16")
        got = H.replay(engine, requests, steps)
        for rid, toks in requests.items():
            close(got[rid], plain_logits(folder, toks), TOL["bfloat16"], f"ordinary/{rid}")
        assert engine.rt.generic_attention_launches == 0 and engine.rt.library_products == 0


def test_recorded_steps_of_a_changing_batch(tmp_path):
    """Three requests decode together from recorded steps while the states go on in their slots and the window moves over pages;
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
    folder = folders[("bavedra-tiny-b", dtype)]
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
    folder = folders[("bavedra-tiny-a", "bfloat16")]
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
