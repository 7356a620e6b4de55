"""The Bavedra design without a GPU: the plain implementation's mechanisms by hand or against a second formulation, the
configuration's keys and refusals, the tensors the parts declare, what the cache manager is asked for."""
import copy
import math

import numpy as np
import pytest

from tests.plain import bavedra_plain as P


def tiny(name="bavedra-tiny-a"):
    from kipp_amd.config import shape_config
    return shape_config(name)


def weights_of(cfg, seed):
    import torch
    from kipp_amd.config import parse_config
    from kipp_amd.engine.model import model_params
    from kipp_amd.weights.random_init import random_tensor
    spec = parse_config(cfg)[1].model_spec()
    return {name: random_tensor(seed, name, p, torch.float32).double().numpy() for name, p in model_params(spec).items()}


# =============================================================================== the plain implementation

def test_rotation_turns_neighbours_and_leaves_the_rest():
    x = np.arange(1.0, 8.0).reshape(1, 1, 7)
    out = P.rotate_neighbours(x, [3], 4, 100.0)
    a, b = 3.0, 3 * 100.0 ** -0.5
    assert np.allclose(out[0, 0], [1 * math.cos(a) - 2 * math.sin(a), 2 * math.cos(a) + 1 * math.sin(a),
                                   3 * math.cos(b) - 4 * math.sin(b), 4 * math.cos(b) + 3 * math.sin(b), 5.0, 6.0, 7.0])
    assert np.allclose(P.rotate_neighbours(x, [0], 4, 100.0), x)
    # a query and a key that are turned by the same distance have the same product
    q, k = np.random.default_rng(0).normal(size=(2, 1, 1, 7))
    one = (P.rotate_neighbours(q, [9], 6, 50.0) * P.rotate_neighbours(k, [4], 6, 50.0)).sum()
    two = (P.rotate_neighbours(q, [25], 6, 50.0) * P.rotate_neighbours(k, [20], 6, 50.0)).sum()
    assert np.isclose(one, two)


def test_window_and_the_added_one():
    """A lone key of score s weighs e^s / (1 + e^s); i sees i - size + 1 .. i; a score far below zero leaves (almost) nothing."""
    q, k, v = np.ones((1, 1, 2)), np.array([[[0.5, 0.5]]]), np.array([[[2.0]]])
    assert np.isclose(P.window_attention_core(q, k, v, 1.0, 5)[0, 0, 0], 2.0 * math.e / (1 + math.e))
    assert abs(P.window_attention_core(q, -100 * k, v, 1.0, 5)[0, 0, 0]) < 1e-12
    rng = np.random.default_rng(0)
    t_len, size = 11, 4
    q, k, v = rng.normal(size=(t_len, 4, 6)), rng.normal(size=(t_len, 2, 6)), rng.normal(size=(t_len, 2, 6))
    out, every = P.window_attention_core(q, k, v, 0.7, size), P.window_attention_core(q, k, v, 0.7, None)
    for i in (0, 3, 4, 10):
        lo = max(0, i - size + 1)
        for at, first in ((out, lo), (every, 0)):
            for h in range(4):
                w = np.exp(k[first:i + 1, h // 2] @ q[i, h] * 0.7)
                assert np.allclose(at[i, h], (w / (1.0 + w.sum())) @ v[first:i + 1, h // 2])


def test_the_values_are_the_keys_before_their_rotation():
    """With a query of zeros every seen key weighs 1 / (n + 1): the result is the sum of the unturned keys."""
    rng = np.random.default_rng(3)
    m = {"heads": 2, "kv_heads": 1, "dim": 4, "vdim": 4, "scale": 0.5, "mask": {"size": 3}, "rot": {"base": 10.0, "dims": 4}}
    w = {"q": np.zeros((8, 5)), "k": rng.normal(size=(4, 5)), "o": np.eye(8)}
    h = rng.normal(size=(6, 5))
    out = P.key_value_attention(w, "", m, h, 1e-5)
    keys = h @ w["k"].T
    for i in range(6):
        seen = keys[max(0, i - 2):i + 1]
        assert np.allclose(out[i], np.tile(seen.sum(0) / (len(seen) + 1), 2))


def test_two_results_are_normed_apart_and_halved():
    rng = np.random.default_rng(4)
    a, b = rng.normal(size=(3, 8)) * 100, rng.normal(size=(3, 8)) * 1e-3
    wa, wb = rng.normal(size=8), rng.normal(size=8)
    out = P.normed_mean(a, b, wa, wb, 1e-5)
    for t in range(3):
        ref = 0.5 * a[t] / math.sqrt(np.mean(a[t] ** 2) + 1e-5) * wa + 0.5 * b[t] / math.sqrt(np.mean(b[t] ** 2) + 1e-5) * wb
        assert np.allclose(out[t], ref)
    assert not np.allclose(out, P.rms_norm(0.5 * (a + b), wa, 1e-5))


def test_causal_filter_by_hand_and_across_a_cut():
    x = np.array([[1.0, 10.0], [2.0, 20.0], [3.0, 30.0], [4.0, 40.0]])
    w, b = np.array([[0.5, 1.0, 2.0], [1.0, 0.0, -1.0]]), np.array([0.25, -1.0])
    out = P.causal_filter(x, w, b)
    assert np.allclose(out[0], [2.25, -11.0]) and np.allclose(out[2], [0.5 + 2.0 + 6.0 + 0.25, 10.0 - 30.0 - 1.0])
    assert np.allclose(P.causal_filter(x[2:], w, b, before=x[:2]), out[2:])
    assert np.allclose(P.causal_filter(x, w) + b, out)


def test_gated_recurrence_against_the_sum_over_earlier_tokens():
    rng = np.random.default_rng(5)
    t_len, width = 9, 6
    u, r, i, lam = rng.normal(size=(t_len, width)), rng.uniform(size=(t_len, width)), rng.uniform(size=(t_len, width)), rng.normal(size=width)
    out, last = P.gated_recurrence(u, r, i, lam)
    a = np.exp(-8.0 * r * np.log1p(np.exp(lam)))
    for t in range(t_len):
        ref = sum(np.prod(a[s + 1:t + 1], axis=0) * np.sqrt(1 - a[s] ** 2) * i[s] * u[s] for s in range(t + 1))
        assert np.allclose(out[t], ref)         # the first token's input too is weighed by sqrt(1 - a^2)
    one, mid = P.gated_recurrence(u[:4], r[:4], i[:4], lam)
    two, end = P.gated_recurrence(u[4:], r[4:], i[4:], lam, state=mid)
    assert np.allclose(np.concatenate([one, two]), out) and np.allclose(end, last)
    ra, ri = rng.normal(size=(2, 3, 3)), rng.normal(size=(2, 3, 3))
    gr, gi = P.block_gates(u, ra, np.zeros((2, 3)), ri, np.ones((2, 3)))
    assert np.allclose(gr[4, 3:], P.sigmoid(ra[1] @ u[4, 3:])) and np.allclose(gi[4, :3], P.sigmoid(ri[0] @ u[4, :3] + 1.0))


def test_state_space_walk_against_the_sum_over_earlier_tokens():
    rng = np.random.default_rng(1)
    t_len, heads, p, groups, n = 8, 4, 3, 2, 5
    x, b, c = rng.normal(size=(t_len, heads, p)), rng.normal(size=(t_len, groups, n)), rng.normal(size=(t_len, groups, n))
    dt, a_log, skip = P.softplus(rng.normal(size=(t_len, heads))), rng.normal(size=heads) * 0.5, rng.normal(size=heads)
    y, s_end = P.state_space_scan(x, b, c, dt, a_log, skip)
    for h in range(heads):
        g = h // 2
        a = np.exp(-np.exp(a_log[h]) * dt[:, h])
        for t in range(t_len):
            ref = skip[h] * x[t, h] + sum(np.prod(a[s + 1:t + 1]) * dt[s, h] * (c[t, g] @ b[s, g]) * x[s, h] for s in range(t + 1))
            assert np.allclose(y[t, h], ref)
    y1, s1 = P.state_space_scan(x[:3], b[:3], c[:3], dt[:3], a_log, skip)
    y2, s2 = P.state_space_scan(x[3:], b[3:], c[3:], dt[3:], a_log, skip, state=s1)
    assert np.allclose(np.concatenate([y1, y2]), y) and np.allclose(s2, s_end)


def test_delta_rule_writes_before_it_reads_and_replaces_what_a_key_held():
    """With beta = g = 1 and unit keys a second write under the same key replaces the first, and a read sees the token's own."""
    k = np.array([[[1.0, 0.0]], [[0.0, 1.0]], [[1.0, 0.0]]])
    v = np.array([[[5.0, 6.0, 7.0]] * 2, [[1.0, 2.0, 3.0]] * 2, [[-1.0, 0.0, 4.0]] * 2])
    ones = np.ones((3, 2))
    o, s = P.delta_scan(k, k, v, ones, ones)
    assert np.allclose(o, v) and np.allclose(s[0], [[-1.0, 0.0, 4.0], [1.0, 2.0, 3.0]])
    o, s = P.delta_scan(k, k, v, 0.5 * ones, 0.25 * ones)
    assert np.allclose(o[0], 0.5 * v[0]) and np.allclose(o[2, 0], 0.5 * 0.25 ** 2 * v[0, 0] + 0.5 * (v[2, 0] - 0.5 * 0.25 ** 2 * v[0, 0]))
    rng = np.random.default_rng(6)
    q, kk, vv = rng.normal(size=(7, 2, 4)), P.unit(rng.normal(size=(7, 2, 4))), rng.normal(size=(7, 4, 3))
    beta, g = rng.uniform(size=(7, 4)), rng.uniform(size=(7, 4))
    o, s = P.delta_scan(q, kk, vv, beta, g)
    o1, s1 = P.delta_scan(q[:3], kk[:3], vv[:3], beta[:3], g[:3])
    o2, s2 = P.delta_scan(q[3:], kk[3:], vv[3:], beta[3:], g[3:], state=s1)
    assert np.allclose(np.concatenate([o1, o2]), o) and np.allclose(s2, s)


def test_router_groups_by_their_largest_correction_and_weights():
    z = np.array([3.0, -3.0, 2.9, 2.8, -0.5, -0.4, -1.0, -1.1])       # groups of two: {0,1} {2,3} {4,5} {6,7}
    s = np.exp(z) / np.exp(z).sum()
    zero = np.zeros(8)
    chosen, weights, _ = P.route(z, zero, 2, 4, 1)
    assert chosen == [0, 1]                                           # the group with the largest single score, not the largest sum
    assert np.allclose(weights, s[[0, 1]] / s[[0, 1]].sum())
    assert P.route(z, zero, 3, 4, 2)[0] == [0, 2, 3]
    corr = zero.copy()
    corr[7] = 2.0                                                     # lifts its group and itself, and not its weight
    chosen, weights, _ = P.route(z, corr, 2, 4, 1)
    assert chosen == [7, 6] and np.allclose(weights, s[[7, 6]] / s[[7, 6]].sum())
    assert P.route(z, np.full(8, -9.0), 2, 4, 1)[0] == [0, 1]         # negative choice scores: the others count as minus infinity
    assert P.route(np.zeros(8), zero, 3, 4, 2)[0] == [0, 1, 2]        # ties: the lower index
    assert P.route(z, zero, 2)[0] == [0, 2]


def test_identity_experts_the_shared_gate_and_the_squared_relu():
    rng = np.random.default_rng(7)
    width, ff = 4, 3
    mlp = {"router": {"experts": 2, "identity": 1, "top": 2}, "expert": {"ff": ff}, "shared": {"ff": 2}}
    w = {"router": np.zeros((3, width)), "correction": np.array([0.0, -1.0, 0.5]), "shared.sg": rng.normal(size=(1, width))}
    for e, n in (("e0", ff), ("e1", ff), ("shared", 2)):
        w.update({f"{e}.gate": rng.normal(size=(n, width)), f"{e}.up": rng.normal(size=(n, width)), f"{e}.down": rng.normal(size=(width, n))})
    h = rng.normal(size=(3, width))
    out = P.routed_ff(w, "", mlp, h)
    gate = 1.0 / (1.0 + np.exp(-(h @ w["shared.sg"].T)))
    # equal scores: the identity expert and expert 0 are chosen, half a weight each
    assert np.allclose(out, 0.5 * h + 0.5 * P.expert_ff(w, "e0.", h) + gate * P.expert_ff(w, "shared.", h))
    del mlp["shared"]
    assert np.allclose(P.routed_ff(w, "", mlp, h), 0.5 * h + 0.5 * P.expert_ff(w, "e0.", h))
    d = {"up": np.array([[1.0, 0.0], [0.0, 1.0]]), "down": np.array([[1.0, 1.0]])}
    assert np.allclose(P.dense_ff(d, "", np.array([[3.0, -2.0]])), [[9.0]])


def test_a_changed_token_reaches_the_positions_the_design_lets_it():
    """Each mixer alone: nothing looks ahead; the recurrences reach every later position, the window only its own length."""
    cfg = tiny()
    only = {}
    for kind in ("rglru", "delta", "parallel"):
        only[kind] = copy.deepcopy(cfg)
        only[kind]["layers"] = [next(l for l in cfg["layers"] if l["type"] == kind)]
    attention = copy.deepcopy(only["parallel"])
    size = attention["layers"][0]["mixer"]["left"]["mask"]["size"]
    tokens = list(np.random.default_rng(4).integers(0, cfg["vocab"], size=45))
    for name, c in list(only.items()) + [("attention", attention)]:
        w = weights_of(c, 3)
        if name == "attention":
            w["l0.mix.right.o"] = np.zeros_like(w["l0.mix.right.o"])
        base = P.forward_whole(c, w, tokens)
        for at in (0, 11):
            changed = list(tokens)
            changed[at] = (changed[at] + 1) % cfg["vocab"]
            moved = np.abs(P.forward_whole(c, w, changed) - base).max(axis=1)
            assert np.all(moved[:at] == 0) and np.all(moved[at:at + size] > 1e-12), name
            assert np.all(moved[at + size:] == 0) if name == "attention" else np.all(moved[at + size:] > 1e-14), name


def test_shared_weights_and_the_embedding_scale():
    """A layer that names another's weights is that layer once more; the residual stream starts at the scaled rows."""
    cfg = tiny()
    w = weights_of(cfg, 5)
    tokens = [3, 9, 1, 77, 20]
    layers = []
    base = P.forward_whole(cfg, w, tokens, layers)
    twice = copy.deepcopy(cfg)
    for layer in twice["layers"]:
        layer.pop("weights_of", None)
    spelled = dict(w)
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            spelled.update({f"l{i}." + name.split(".", 1)[1]: t for name, t in w.items() if name.startswith(f"l{layer['weights_of']}.")})
    assert np.array_equal(P.forward_whole(twice, spelled, tokens), base) and len(layers) == len(cfg["layers"])
    still = copy.deepcopy(cfg)
    still["layers"] = [dict(cfg["layers"][5], mlp=None)]
    quiet = {name.replace("l5.", "l0."): (np.zeros_like(t) if name == "l5.mix.o" else t) for name, t in w.items()}
    out = []
    P.forward_whole(still, quiet, tokens, out)
    assert np.allclose(out[0], w["embed"][tokens] * cfg["embedding"]["scale"])


# =============================================================================== configuration, tensors, cache needs

def test_configuration_keys_and_refusals():
    from kipp_amd.config import ConfigError, parse_config
    cfg = tiny()
    family, typed = parse_config(cfg)
    assert family.name == "Bavedra" and typed.to_dict()["layers"] == cfg["layers"] and typed.to_dict()["embedding"] == {"scale": 7.5}
    spec = typed.model_spec()
    assert [layer.block for layer in spec.layers] == ["pre_norm"] * 3 + ["pre_norm_mixer"]
    assert [run.layer for run in spec.order] == [0, 1, 2, 1, 0, 3] and all(run.cache_of is None for run in spec.order)
    side = spec.layers[1].part("mixer")
    assert side.kind == "parallel_mixer" and (side.left_scale, side.right_scale) == (0.5, 0.5)
    assert side.left.keys_as_values and side.left.sink and side.left.window == 21 and not side.left.plain
    assert side.left.position.pairing == "interleaved" and side.left.position.rotary_dim == 16
    assert side.left_norm.prefix == "l1.mix.left.out" and side.left_norm.eps == 1e-5 and side.right.norm_groups == 2
    routed = spec.layers[1].part("ffn")
    assert routed.router == "softmax" and routed.groups == (3, 2) and routed.group_score == "top1" and routed.identity == 2 and routed.choices == 9
    assert routed.shared_gate_name == "shared.sg" and routed.gate_name == "gate" and spec.layers[2].part("ffn").shared_gate_name is None
    assert spec.layers[0].part("ffn").kind == "dense_mlp" and spec.layers[0].part("ffn").activation == "relu2"
    assert not spec.head.tied and spec.embedding.scale == 7.5

    plain = copy.deepcopy(cfg)              # what may be left out
    plain["layers"][1]["mlp"]["router"].pop("groups")
    plain["layers"][1]["mlp"]["router"].pop("identity")
    plain["layers"] = plain["layers"][:2]
    routed = parse_config(plain)[1].model_spec().layers[1].part("ffn")
    assert routed.groups is None and routed.identity == 0

    def broken(change):
        bad = copy.deepcopy(cfg)
        change(bad)
        with pytest.raises(ConfigError):
            parse_config(bad)
    broken(lambda c: c["layers"][1]["mixer"]["left"].update(softcap=3.0))              # a key the design does not have
    broken(lambda c: c["layers"][0].update(type="attention"))
    broken(lambda c: c["layers"][1]["mixer"]["left"].update(vdim=16))                  # the values are the keys
    broken(lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7))
    broken(lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=0))
    broken(lambda c: c["layers"][1]["mixer"]["right"].update(norm_groups=5))
    broken(lambda c: c["layers"][1]["mixer"].update(left_scale=1.0))
    broken(lambda c: c["layers"][0]["mixer"].update(kv_heads=3))                       # does not divide the heads
    broken(lambda c: c["layers"][2]["mixer"].update(blocks=5))
    broken(lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=2))        # 9 outputs in 2 groups
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(top=7))                    # more than the kept groups hold
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(scale=2.0))
    broken(lambda c: c["layers"][3].update(weights_of=4))                              # not an earlier layer
    broken(lambda c: c["layers"][3].update(weights_of=0))                              # another kind of layer
    broken(lambda c: c["layers"][3]["mixer"]["right"].update(conv=3))                  # sizes that are not the other layer's
    broken(lambda c: c.pop("embedding"))
    broken(lambda c: c.update(loop={"start": 0, "stop": 1, "times": 2}))


def test_specs_of_the_new_mechanisms_refuse_what_they_cannot_be():
    from kipp_amd.config import AttentionSpec, ConfigError, DenseMLPSpec, ParallelMixerSpec, RMSNormSpec, RoutedMLPSpec
    for bad in (dict(v_head_dim=8), dict(own_kv=False), dict(v_norm_eps=1e-5), dict(v_mix="source")):
        with pytest.raises(ConfigError):
            AttentionSpec(hidden_size=16, num_heads=2, num_kv_heads=1, head_dim=16, keys_as_values=True, **bad)
    with pytest.raises(ConfigError):
        ParallelMixerSpec(left=None, right=None, left_norm=RMSNormSpec(16, 1e-5))
    with pytest.raises(ConfigError):
        DenseMLPSpec(hidden_size=16, intermediate_size=8, activation="tanh")
    base = dict(hidden_size=16, experts=4, top=2, expert_size=8)
    for bad in (dict(identity=-1), dict(group_score="mean"), dict(groups=(4, 1), identity=1), dict(shared_gate_name="sg"),
                dict(identity=2, weigh_input=True, gate_name="gate"), dict(top=5)):
        with pytest.raises(ConfigError):
            RoutedMLPSpec(**dict(base, **bad))
    assert RoutedMLPSpec(**dict(base, top=5, identity=1)).choices == 5


def test_tensor_names_and_cache_needs():
    from kipp_amd.cache.needs import KVNeed
    from kipp_amd.config import parse_config
    from kipp_amd.engine.model import cache_bytes_per_page, model_params
    from kipp_amd.parts import part_class
    spec = parse_config(tiny())[1].model_spec()
    names = model_params(spec)
    for name, shape in (("embed", (180, 64)), ("head", (180, 64)), ("final.norm", (64,)), ("l0.norm1", (64,)), ("l0.norm2", (64,)),
                        ("l0.mix.q", (32, 64)), ("l0.mix.q.conv", (32, 3)), ("l0.mix.v.conv", (96, 3)), ("l0.mix.b", (4, 64)), ("l0.mix.norm", (24,)),
                        ("l0.mlp.up", (160, 64)), ("l0.mlp.down", (64, 160)), ("l1.mix.left.q", (128, 64)), ("l1.mix.left.k", (64, 64)),
                        ("l1.mix.left.o", (64, 128)), ("l1.mix.left.out", (64,)), ("l1.mix.right.out", (64,)), ("l1.mix.right.in", (2 * 64 + 2 * 48 + 4, 64)),
                        ("l1.mix.right.conv.b", (160,)), ("l1.mlp.router", (9, 64)), ("l1.mlp.correction", (9,)), ("l1.mlp.e6.gate", (32, 64)),
                        ("l1.mlp.shared.sg", (1, 64)), ("l1.mlp.shared.down", (64, 48)), ("l2.mix.ra", (3, 32, 32)), ("l2.mix.lam", (96,)),
                        ("l5.mix.y.b", (40,))):
        assert tuple(names[name].shape) == shape, name
    assert not any(name.startswith(("l3.", "l4.")) for name in names)
    assert not {"l1.mix.left.v", "l1.mlp.e7.up", "l0.mlp.gate", "l2.mlp.shared.sg", "l5.norm2", ""} & set(names)
    needs = [part_class("mixer", layer.part("mixer").kind) for layer in spec.layers]
    assert needs[1].need_of(spec.layers[1].part("mixer")) == KVNeed(2, 32, window=21, v_head_dim=None)
    assert cache_bytes_per_page(spec, 16, 2) == 2 * 16 * 2 * 2 * (32 + 32)      # two runs of the layer, each with a cache of its own


def test_plain_runs_a_tiny_model_and_reports_margins():
    cfg = tiny("bavedra-tiny-b")
    w = weights_of(cfg, 1)
    layers, margins = [], []
    logits = P.forward_whole(cfg, w, [1, 5, 9, 2, 7], layers, margins)
    assert logits.shape == (5, cfg["vocab"]) and len(layers) == 6 and np.isfinite(logits).all()
    assert len(margins) == 3 * 5 and min(margins) >= 0
