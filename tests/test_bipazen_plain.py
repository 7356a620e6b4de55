"""The Bipazen design without a GPU: the plain implementation's mechanisms by hand or against a second formulation, the
configuration's keys and refusals, the tensors the parts declare, what the cache manager is asked for."""
import copy
import math

import numpy as np
import pytest

from tests.plain import bipazen_plain as P


def tiny(name="bipazen-tiny-a"):
    from kipp_amd.config import shape_config
    return shape_config(name)


def weights_of(cfg, seed, sharpen=True):
    """Random tensors of a configuration as float64 arrays, by name; long memories and few keys that carry a row's softmax."""
    import torch
    from kipp_amd.config import parse_config
    from kipp_amd.engine.model import model_params
    from kipp_amd.weights.random_init import random_tensor
    spec = parse_config(cfg)[1].model_spec()
    w = {name: random_tensor(seed, name, p, torch.float32).double().numpy() for name, p in model_params(spec).items()}
    if sharpen:
        for name in w:
            if name.endswith(".mix.lam"):
                w[name] = w[name] - 5.0
            elif name.endswith((".mix.q", ".mix.uk", ".mix.dkv", ".mlp.router")):
                w[name] = w[name] * 8.0
    return w


# =============================================================================== the plain implementation

def test_activations_by_hand():
    assert np.isclose(P.gelu_tanh(1.5), 0.5 * 1.5 * (1 + math.tanh(math.sqrt(2 / math.pi) * (1.5 + 0.044715 * 1.5 ** 3))))
    assert np.isclose(P.gelu_tanh(np.array(-20.0)), 0.0) and np.isclose(P.gelu_tanh(np.array(20.0)), 20.0)
    assert np.isclose(P.silu(2.0), 2.0 / (1.0 + math.exp(-2.0)))
    assert np.isclose(P.softplus(0.3), math.log(1.0 + math.exp(0.3)))


def test_causal_filter_by_hand_and_across_a_cut():
    x = np.array([[1.0, 10.0], [2.0, 20.0], [3.0, 30.0], [4.0, 40.0]])
    w = np.array([[0.5, 1.0, 2.0], [1.0, 0.0, -1.0]])
    b = np.array([0.25, -1.0])
    out = P.causal_filter(x, w, b)
    assert np.allclose(out[0], [2.0 * 1 + 0.25, -10.0 - 1.0])
    assert np.allclose(out[2], [0.5 * 1 + 1.0 * 2 + 2.0 * 3 + 0.25, 10.0 - 30.0 - 1.0])
    assert np.allclose(P.causal_filter(x[2:], w, b, before=x[:2]), out[2:])


def test_gates_use_each_parts_own_matrix():
    rng = np.random.default_rng(0)
    u = rng.normal(size=(3, 6))
    ra, ri = rng.normal(size=(3, 2, 2)), rng.normal(size=(3, 2, 2))
    rb, ib = rng.normal(size=(3, 2)), rng.normal(size=(3, 2))
    r, i = P.block_gates(u, ra, rb, ri, ib)
    for t in range(3):
        for c in range(6):
            b, o = divmod(c, 2)
            assert np.isclose(r[t, c], P.sigmoid(ra[b, o, 0] * u[t, 2 * b] + ra[b, o, 1] * u[t, 2 * b + 1] + rb[b, o]))
            assert np.isclose(i[t, c], P.sigmoid(ri[b, o, 0] * u[t, 2 * b] + ri[b, o, 1] * u[t, 2 * b + 1] + ib[b, o]))


def test_gated_recurrence_against_the_sum_over_earlier_tokens():
    """S_t = sum_{s <= t} (prod_{s < j <= t} a_j) sqrt(1 - a_s^2) i_s u_s (the first token like every other), and a cut with the
    state handed on."""
    rng = np.random.default_rng(1)
    t_len, width = 9, 4
    u, r, i = rng.normal(size=(t_len, width)), rng.uniform(size=(t_len, width)), rng.uniform(size=(t_len, width))
    lam = rng.normal(size=width) - 3.0
    a = np.exp(-8.0 * r * np.log1p(np.exp(lam)))
    out, last = P.gated_recurrence(u, r, i, lam)
    for t in range(t_len):
        ref = sum(np.prod(a[s + 1:t + 1], axis=0) * np.sqrt(1 - a[s] ** 2) * i[s] * u[s] for s in range(t + 1))
        assert np.allclose(out[t], ref)
    assert np.allclose(out[0], np.sqrt(1 - a[0] ** 2) * i[0] * u[0])
    o1, s1 = P.gated_recurrence(u[:4], r[:4], i[:4], lam)
    o2, s2 = P.gated_recurrence(u[4:], r[4:], i[4:], lam, state=s1)
    assert np.allclose(np.concatenate([o1, o2]), out) and np.allclose(s2, last)


def test_state_space_walk_against_the_sum_over_earlier_tokens():
    rng = np.random.default_rng(1)
    t_len, heads, p, groups, n = 9, 4, 3, 2, 5
    x, b, c = rng.normal(size=(t_len, heads, p)), rng.normal(size=(t_len, groups, n)), rng.normal(size=(t_len, groups, n))
    dt = P.softplus(rng.normal(size=(t_len, heads)))
    a_log, skip = rng.normal(size=heads) * 0.5, rng.normal(size=heads)
    y, s_end = P.state_space_scan(x, b, c, dt, a_log, skip)
    for h in range(heads):
        g = h // (heads // groups)
        a = np.exp(-np.exp(a_log[h]) * dt[:, h])
        for t in range(t_len):
            ref = skip[h] * x[t, h]
            for s in range(t + 1):
                ref = ref + np.prod(a[s + 1:t + 1]) * dt[s, h] * (c[t, g] @ b[s, g]) * x[s, h]
            assert np.allclose(y[t, h], ref)
    y1, s1 = P.state_space_scan(x[:4], b[:4], c[:4], dt[:4], a_log, skip)
    y2, s2 = P.state_space_scan(x[4:], b[4:], c[4:], dt[4:], a_log, skip, state=s1)
    assert np.allclose(np.concatenate([y1, y2]), y) and np.allclose(s2, s_end)


def test_rotation_turns_halves_by_the_position():
    x = np.arange(1.0, 5.0).reshape(1, 1, 4)
    out = P.rotate(x, [3], 4, 100.0)
    a, b = 3.0, 3.0 * 100.0 ** -0.5
    assert np.allclose(out[0, 0], [1 * math.cos(a) - 3 * math.sin(a), 2 * math.cos(b) - 4 * math.sin(b),
                                   3 * math.cos(a) + 1 * math.sin(a), 4 * math.cos(b) + 2 * math.sin(b)])
    assert np.allclose(P.rotate(x, [0], 4, 100.0), x)


def test_latent_attention_against_its_absorbed_form():
    """Scores against the cached row [c | kr] with each head's query carried into the latent's space, values carried back from
    the weighted sum of rows: the same numbers, head by head and position by position."""
    rng = np.random.default_rng(3)
    t_len, width, eps = 7, 10, 1e-5
    m = {"heads": 3, "dim": 4, "rot_dim": 6, "vdim": 5, "kv_rank": 8, "scale": 0.4, "rot": {"base": 50.0, "dims": 6}}
    hds, d, dr, dv, rank = 3, 4, 6, 5, 8
    w = {"q": rng.normal(size=(hds * (d + dr), width)), "dkv": rng.normal(size=(rank + dr, width)), "dkv.norm": rng.normal(size=rank),
         "uk": rng.normal(size=(hds * d, rank)), "uv": rng.normal(size=(hds * dv, rank)), "g": rng.normal(size=(hds * dv, width)),
         "o": np.eye(hds * dv)}
    h = rng.normal(size=(t_len, width))
    got = P.latent_attention(w, "", m, h, list(range(t_len)), eps)
    down = h @ w["dkv"].T
    c = down[:, :rank] / np.sqrt(np.mean(down[:, :rank] ** 2, axis=1, keepdims=True) + eps) * w["dkv.norm"]
    turn = lambda v, p: P.rotate(v.reshape(1, 1, -1), [p], 6, 50.0).reshape(-1)
    for t in range(t_len):
        q = w["q"] @ h[t]
        for k in range(hds):
            part = q[k * (d + dr):(k + 1) * (d + dr)]
            lat, rot = w["uk"][k * d:(k + 1) * d].T @ part[:d], turn(part[d:], t)
            s = np.array([0.4 * (lat @ c[j] + rot @ turn(down[j, rank:], j)) for j in range(t + 1)])
            p = np.exp(s - s.max()) / np.exp(s - s.max()).sum()
            o = w["uv"][k * dv:(k + 1) * dv] @ (p @ c[:t + 1])
            assert np.allclose(got[t, k * dv:(k + 1) * dv], o * P.sigmoid(w["g"][k * dv:(k + 1) * dv] @ h[t]))


def test_router_takes_scores_as_weights_of_the_experts_inputs():
    z = np.array([0.3, -1.0, 2.0, 0.3])
    chosen, weights, margin = P.route(z, 2)
    assert chosen == [2, 0] and np.allclose(weights, P.sigmoid(np.array([2.0, 0.3]))) and margin == 0.0
    assert P.route(z, 4)[0] == [2, 0, 3, 1]
    w = {"router": np.array([[1.0, 0.0], [-1.0, 0.0]]), "e0.gate": np.array([[1.0, 2.0]]), "e0.up": np.array([[0.5, -1.0]]),
         "e0.down": np.array([[2.0], [3.0]]), "e1.gate": np.ones((1, 2)), "e1.up": np.ones((1, 2)), "e1.down": np.ones((2, 1))}
    h = np.array([[0.7, -0.2]])
    out = P.routed_ff(w, "", {"router": {"experts": 2, "top": 1}}, h)
    s = 1 / (1 + math.exp(-0.7))
    gate, up = s * (0.7 - 0.4), s * (0.35 + 0.2)
    assert np.allclose(out, np.array([[2.0, 3.0]]) * (gate / (1 + math.exp(-gate))) * up)
    # not the same as a weight on the result: the expert is not linear
    assert not np.allclose(out, s * P.expert(w, "e0.", h))


def test_a_changed_token_reaches_every_later_position_and_none_before():
    """Each mixer alone: position 0 shows at the last of 40 positions through the memory or the keys; nothing looks ahead."""
    cfg = tiny()
    for kind in ("mamba2", "rglru", "latent_attention"):
        only = copy.deepcopy(cfg)
        only["layers"] = [next(l for l in cfg["layers"] if l["type"] == kind)]
        w = weights_of(only, 3)
        tokens = list(np.random.default_rng(4).integers(0, cfg["vocab"], size=40))
        base = P.forward_whole(only, w, tokens)
        for at in (0, 17):
            changed = list(tokens)
            changed[at] = (changed[at] + 1) % cfg["vocab"]
            moved = np.abs(P.forward_whole(only, w, changed) - base).max(axis=1)
            assert np.all(moved[:at] == 0) and np.all(moved[at:] > 1e-12), kind


def test_shared_weights_and_scales():
    """A layer that names another's weights is that layer once more; a scale multiplies a sublayer's result column by column."""
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
    assert np.array_equal(P.forward_whole(twice, spelled, tokens), base)
    still = dict(w)
    still["l0.ls1"] = w["l0.ls1"] * np.where(np.arange(cfg["width"]) == 3, 0.0, 1.0)
    one = copy.deepcopy(cfg)
    one["layers"] = [dict(cfg["layers"][0], mlp=None)]
    x, y = [], []
    P.forward_whole(one, w, tokens, x)
    P.forward_whole(one, still, tokens, y)
    assert np.allclose(y[0][:, 3], w["embed"][tokens][:, 3]) and not np.allclose(x[0][:, 3], y[0][:, 3])
    assert np.allclose(np.delete(x[0], 3, axis=1), np.delete(y[0], 3, axis=1)) and len(layers) == len(cfg["layers"])


# =============================================================================== configuration, tensors, cache needs

def test_configuration_keys_and_refusals():
    from kipp_amd.config import ConfigError, parse_config
    cfg = tiny()
    family, typed = parse_config(cfg)
    assert family.name == "Bipazen" and typed.to_dict()["layers"] == cfg["layers"]
    spec = typed.model_spec()
    assert [layer.block for layer in spec.layers] == ["scaled_pre_norm"] * 3 + ["scaled_pre_norm_mixer"]
    assert [run.layer for run in spec.order] == [0, 1, 2, 1, 2, 3] and all(run.cache_of is None for run in spec.order)
    lat = spec.layers[2].part("mixer")
    assert lat.q_rank is None and lat.gate_each and lat.window is None and lat.position.pairing == "half" and lat.row == 48
    lru = spec.layers[1].part("mixer")
    assert (lru.width, lru.blocks, lru.conv_taps, lru.factor) == (96, 3, 4, 8.0)
    ffn = spec.layers[0].part("ffn")
    assert ffn.router == "sigmoid" and not ffn.renormalize and ffn.weigh_input and ffn.gate_name == "gate" and ffn.correction_name is None
    assert spec.head.tied and spec.embedding.scale == 1.0

    def broken(change):
        bad = copy.deepcopy(cfg)
        change(bad)
        with pytest.raises(ConfigError):
            parse_config(bad)
    broken(lambda c: c["layers"][0]["mixer"].update(clamp=3.0))                        # a key the design does not have
    broken(lambda c: c["layers"][0].update(type="attention"))
    broken(lambda c: c["layers"][0]["mixer"].update(norm_groups=5))
    broken(lambda c: c["layers"][1]["mixer"].update(blocks=5))                         # does not divide the width
    broken(lambda c: c["layers"][2]["mixer"]["rot"].update(dims=7))
    broken(lambda c: c["layers"][2]["mixer"].update(mask={"size": 9}))
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=7))                    # more than there are experts
    broken(lambda c: c["layers"][0]["mlp"].update(shared={"ff": 8}))
    broken(lambda c: c["layers"][3].update(weights_of=4))                              # not an earlier layer
    broken(lambda c: c["layers"][3].update(weights_of=0))                              # another kind of layer
    broken(lambda c: c["layers"][3]["mixer"].update(conv=3))                           # sizes that are not the other layer's
    broken(lambda c: c.update(embedding={"scale": 2.0}))


def test_specs_of_the_new_mechanisms_refuse_what_they_cannot_be():
    from kipp_amd.config import ConfigError, GatedRecurrenceSpec, RoutedMLPSpec
    for bad in (dict(width=30, blocks=4, conv_taps=3), dict(width=32, blocks=4, conv_taps=17), dict(width=32, blocks=4, conv_taps=3, factor=0.0)):
        with pytest.raises(ConfigError):
            GatedRecurrenceSpec(hidden_size=16, **bad)
    with pytest.raises(ConfigError):
        RoutedMLPSpec(hidden_size=16, experts=4, top=2, expert_size=8, weigh_input=True)           # no gate
    with pytest.raises(ConfigError):
        RoutedMLPSpec(hidden_size=16, experts=4, top=2, expert_size=8, renormalize=False)          # softmax router


def test_tensor_names_and_cache_needs():
    from kipp_amd.cache.needs import KVNeed
    from kipp_amd.config import parse_config
    from kipp_amd.engine.model import cache_bytes_per_page, model_params
    spec = parse_config(tiny())[1].model_spec()
    names = model_params(spec)
    for name, shape in (("embed", (160, 64)), ("final.norm", (64,)), ("l0.norm1", (64,)), ("l0.norm2", (64,)), ("l0.ls1", (64,)), ("l0.ls2", (64,)),
                        ("l0.mix.in", (2 * 64 + 2 * 48 + 4, 64)), ("l0.mix.conv", (160, 4)), ("l0.mix.D", (4,)), ("l1.mix.y", (96, 64)),
                        ("l1.mix.y.b", (96,)), ("l1.mix.x.b", (96,)), ("l1.mix.conv", (96, 4)), ("l1.mix.ra", (3, 32, 32)), ("l1.mix.ri.b", (3, 32)),
                        ("l1.mix.lam", (96,)), ("l1.mix.o", (64, 96)), ("l2.mix.q", (96, 64)), ("l2.mix.dkv", (48, 64)), ("l2.mix.dkv.norm", (40,)),
                        ("l2.mix.uk", (64, 40)), ("l2.mix.uv", (96, 40)), ("l2.mix.g", (96, 64)), ("l2.mlp.router", (5, 64)),
                        ("l2.mlp.e4.gate", (32, 64)), ("l2.mlp.e4.down", (64, 32)), ("l5.ls1", (64,))):
        assert tuple(names[name].shape) == shape, name
    assert not any(name.startswith(("l3.", "l4.", "head")) for name in names) and "l5.norm2" not in names and "l5.ls2" not in names
    from kipp_amd.parts import part_class
    lat = spec.layers[2].part("mixer")
    assert part_class("mixer", lat.kind).need_of(lat) == KVNeed(1, 48, window=None, v_head_dim=0)
    assert cache_bytes_per_page(spec, 16, 2) == 2 * 16 * 2 * 48         # two runs of the layer, each with a cache of its own


def test_plain_runs_a_tiny_model_and_reports_margins():
    cfg = tiny("bipazen-tiny-b")
    w = weights_of(cfg, 1)
    layers, margins = [], []
    logits = P.forward_whole(cfg, w, [1, 5, 9, 2, 7], layers, margins)
    assert logits.shape == (5, cfg["vocab"]) and len(layers) == 7 and np.isfinite(logits).all()
    assert len(margins) == 4 * 5 and min(margins) >= 0
