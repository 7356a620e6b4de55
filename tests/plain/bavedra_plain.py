"""The plain implementation of the Bavedra decoder: whole sequences, no cache, no pages, no batching, one function for
each mechanism, NumPy float64.  It shares no code with `kipp_amd`; model folders are read with the `safetensors` package.

Notation: a sequence has T tokens at positions 0 .. T-1, X [T, width] is the residual stream, N(x; w) = x / sqrt(mean
x^2 + eps) * w.

    input            X = scale * embed[tokens]
    layer            X += mixer(N(X; norm1));  X += ff(N(X; norm2))     (a layer may have no ff; a layer may name another whose
                     tensors it uses)
    rglru            y = gelu_tanh(Wy h + by);  u = filter(Wx h + bx) + b;  in every block of u: r = sigmoid(Ra u + ba),
                     i = sigmoid(Ri u + bi);  log a = -8 r softplus(lam);  S_t = a S_(t-1) + sqrt(1 - a^2) i u;  Wo (S * y)
    parallel         (N(left(h); left.out) + N(right(h); right.out)) / 2
      left           q, k = Wq h, Wk h;  v = k;  then the first `dims` numbers of every q and k head turned by the position,
                     neighbours paired;  i sees j when 0 <= i - j < size;  s_ij = scale q_i . k_j;
                     p_ij = e^s_ij / (1 + sum_j e^s_ij);  o_i = sum_j p_ij v_j;  Wo
      right          [z | x | B | C | dt] = W_in h;  x, B, C through a causal filter a channel (with bias) and silu;
                     dt = softplus(dt + dt_bias);  S_t = exp(-exp(A_h) dt) S_(t-1) + dt B_t x_t^T;  y_t = S_t^T C_t + D_h x_t;
                     y * silu(z), then N in `norm_groups` equal parts (times .norm), then Wo
    delta            q, k, v = silu(filter(Wq h)), silu(filter(Wk h)), silu(filter(Wv h));  q, k a head over sqrt(sum x^2 + 1e-6),
                     q also over sqrt(dim);  beta = sigmoid(Wb h), g = exp(-exp(A_h) softplus(Wa h + dt_h));
                     S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q;
                     every head of o through N(.; norm), times silu(Wg h); Wo
    dense ff         Wd relu(Wu h)^2
    routed ff        s = softmax(Wr h) over experts and identity experts; choice scores c = s + correction; the outputs in
                     `count` groups of neighbours, a group's score its largest c, only the `keep` best groups stay; the `top`
                     largest c among them are chosen; weights s / (sum of the chosen s + 1e-20);
                     sum of weight_e E_e(h), E_e(h) = Wd_e (silu(Wg_e h) * Wu_e h), or h itself for an identity expert;
                     plus sigmoid(W_sg h) times a shared expert of the same form
    output           logits = head N(X; final.norm)
"""
from __future__ import annotations

import json
import math
import os

import numpy as np

DTYPE = np.float64
RECURRENCE_FACTOR = 8.0
UNIT_EPS = 1e-6         # inside the root of the unit norm of the delta rule's queries and keys
ROUTE_EPS = 1e-20       # added to the sum of the chosen experts' scores


def array(x):
    return np.asarray(x, dtype=DTYPE)


def linear(x, w, b=None):
    y = array(x) @ array(w).T
    return y if b is None else y + array(b)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return np.logaddexp(0.0, z)


def rms_norm(x, w, eps):
    x = array(x)
    y = x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)
    return y if w is None else y * array(w)


def causal_filter(x, taps_w, bias=None, before=None):
    """x [T, C], taps_w [C, taps] (the last column weighs the current token's input), zeros (or `before`
    [taps - 1, C]) ahead of the first token."""
    x, taps_w = array(x), array(taps_w)
    taps = taps_w.shape[1]
    ahead = np.zeros((taps - 1, x.shape[1]), dtype=DTYPE) if before is None else array(before)
    full = np.concatenate([ahead, x], axis=0)
    out = np.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(taps):
            out[t] += taps_w[:, j] * full[t + j]
    return out if bias is None else out + array(bias)


# ----------------------------------------------------------------------------- rglru

def block_gates(u, ra, ra_b, ri, ri_b):
    """u [T, width] in len(ra) equal blocks -> (r, i) [T, width]: sigmoid of a square matrix of each block's own, with a bias."""
    width = u.shape[1]
    size = width // len(ra)
    r, i = np.zeros_like(u), np.zeros_like(u)
    for b in range(len(ra)):
        part = slice(b * size, (b + 1) * size)
        r[:, part] = sigmoid(linear(u[:, part], ra[b], ra_b[b]))
        i[:, part] = sigmoid(linear(u[:, part], ri[b], ri_b[b]))
    return r, i


def gated_recurrence(u, r, i, lam, state=None):
    """log a = -8 r softplus(lam); S_t = a_t S_(t-1) + sqrt(1 - a_t^2) i_t u_t, channel by channel.  Returns (S of every token, the last S)."""
    log_a = -RECURRENCE_FACTOR * r * softplus(array(lam))
    a = np.exp(log_a)
    x = np.sqrt(-np.expm1(2.0 * log_a)) * i * u
    s = np.zeros(u.shape[1], dtype=DTYPE) if state is None else np.array(state, dtype=DTYPE)
    out = np.zeros_like(u)
    for t in range(u.shape[0]):
        s = a[t] * s + x[t]
        out[t] = s
    return out, s


def recurrent_mixer(w, p, m, h, eps):
    y = gelu_tanh(linear(h, w[p + "y"], w[p + "y.b"]))
    u = causal_filter(linear(h, w[p + "x"], w[p + "x.b"]), w[p + "conv"], w[p + "conv.b"])
    assert u.shape[1] == m["width"] and w[p + "conv"].shape[1] == m["conv"] and len(w[p + "ra"]) == m["blocks"]
    r, i = block_gates(u, w[p + "ra"], w[p + "ra.b"], w[p + "ri"], w[p + "ri.b"])
    s, _ = gated_recurrence(u, r, i, w[p + "lam"])
    return linear(s * y, w[p + "o"])


# ----------------------------------------------------------------------------- parallel

def rotate_neighbours(x, positions, dims, base):
    """x [T, heads, d]: numbers 2i and 2i + 1 of every head turned by position * base^(-2i / dims), i < dims / 2."""
    x = np.array(x, dtype=DTYPE)
    for i in range(dims // 2):
        angle = array(positions) * float(base) ** (-2.0 * i / dims)
        cos, sin = np.cos(angle)[:, None], np.sin(angle)[:, None]
        u, v = x[..., 2 * i].copy(), x[..., 2 * i + 1].copy()
        x[..., 2 * i] = u * cos - v * sin
        x[..., 2 * i + 1] = v * cos + u * sin
    return x


def window_attention_core(q, k, v, scale, size):
    """q [T, H, d], k and v [T, G, .]; i sees j when 0 <= i - j < size (None: every j <= i); one is added to the
    softmax's denominator."""
    t_len, heads, _ = q.shape
    rep = heads // k.shape[1]
    out = np.zeros((t_len, heads, v.shape[2]), dtype=DTYPE)
    for i in range(t_len):
        lo = 0 if size is None else max(0, i - size + 1)
        for h in range(heads):
            g = h // rep
            s = (k[lo:i + 1, g] @ q[i, h]) * scale
            top = max(s.max(), 0.0)
            e = np.exp(s - top)
            out[i, h] = (e / (math.exp(-top) + e.sum())) @ v[lo:i + 1, g]
    return out


def key_value_attention(w, p, m, h, eps):
    """The left mixer: the values are the keys before their rotation."""
    t_len = h.shape[0]
    heads, groups, d = m["heads"], m["kv_heads"], m["dim"]
    assert m["vdim"] == d
    q = linear(h, w[p + "q"]).reshape(t_len, heads, d)
    k = linear(h, w[p + "k"]).reshape(t_len, groups, d)
    v = k.copy()
    rot = m["rot"]
    q, k = (rotate_neighbours(x, range(t_len), rot["dims"], rot["base"]) for x in (q, k))
    o = window_attention_core(q, k, v, m["scale"], (m.get("mask") or {}).get("size"))
    return linear(o.reshape(t_len, heads * d), w[p + "o"])


def state_space_scan(x, b, c, dt, a_log, d_skip, state=None):
    """x [T, H, P], b and c [T, G, N], dt [T, H] (after softplus): S_t = exp(-exp(A_h) dt) S_(t-1) + dt B_t x_t^T,
    y_t = S_t^T C_t + D_h x_t.  Returns (y [T, H, P], S [H, N, P])."""
    t_len, heads, width = x.shape
    rep = heads // b.shape[1]
    s = np.zeros((heads, b.shape[2], width), dtype=DTYPE) if state is None else np.array(state, dtype=DTYPE)
    y = np.zeros((t_len, heads, width), dtype=DTYPE)
    for t in range(t_len):
        for h in range(heads):
            g = h // rep
            s[h] = math.exp(-math.exp(a_log[h]) * dt[t, h]) * s[h] + dt[t, h] * np.outer(b[t, g], x[t, h])
            y[t, h] = s[h].T @ c[t, g] + d_skip[h] * x[t, h]
    return y, s


def state_space_mixer(w, p, m, h, eps):
    t_len = h.shape[0]
    heads, vd, n, groups = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = heads * vd
    proj = linear(h, w[p + "in"])
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * groups * n], proj[:, 2 * inner + 2 * groups * n:]
    assert dt.shape[1] == heads and w[p + "conv"].shape[1] == m["conv"]
    xbc = silu(causal_filter(xbc, w[p + "conv"], w[p + "conv.b"]))
    x = xbc[:, :inner].reshape(t_len, heads, vd)
    b = xbc[:, inner:inner + groups * n].reshape(t_len, groups, n)
    c = xbc[:, inner + groups * n:].reshape(t_len, groups, n)
    dt = softplus(dt + array(w[p + "dt_bias"]))
    y, _ = state_space_scan(x, b, c, dt, array(w[p + "A_log"]), array(w[p + "D"]))
    y = y.reshape(t_len, inner) * silu(z)
    parts = m["norm_groups"]
    y = rms_norm(y.reshape(t_len, parts, inner // parts), None, eps).reshape(t_len, inner) * array(w[p + "norm"])
    return linear(y, w[p + "o"])


def normed_mean(left, right, w_left, w_right, eps):
    """Half the sum of two results, each normed over its whole width first."""
    return 0.5 * (rms_norm(left, w_left, eps) + rms_norm(right, w_right, eps))


def parallel_mixer(w, p, m, h, eps):
    return normed_mean(key_value_attention(w, p + "left.", m["left"], h, eps), state_space_mixer(w, p + "right.", m["right"], h, eps),
                       w[p + "left.out"], w[p + "right.out"], eps)


# ----------------------------------------------------------------------------- delta

def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + UNIT_EPS)


def delta_scan(q, k, v, beta, g, state=None):
    """q, k [T, G, d] (unit vectors, q scaled), v [T, H, dv], beta and g [T, H]; head h reads q/k head h // (H / G).
    Returns (o [T, H, dv], S [H, d, dv])."""
    t_len, heads, dv = v.shape
    rep = heads // k.shape[1]
    s = np.zeros((heads, k.shape[2], dv), dtype=DTYPE) if state is None else np.array(state, dtype=DTYPE)
    out = np.zeros((t_len, heads, dv), dtype=DTYPE)
    for t in range(t_len):
        for h in range(heads):
            kt, qt = k[t, h // rep], q[t, h // rep]
            s[h] = g[t, h] * s[h]
            u = beta[t, h] * (v[t, h] - s[h].T @ kt)
            s[h] = s[h] + np.outer(kt, u)
            out[t, h] = s[h].T @ qt
    return out, s


def delta_mixer(w, p, m, h, eps):
    t_len = h.shape[0]
    heads, groups, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_filter(linear(h, w[p + n]), w[p + n + ".conv"])) for n in ("q", "k", "v"))
    q, k, v = q.reshape(t_len, groups, d), k.reshape(t_len, groups, d), v.reshape(t_len, heads, dv)
    beta = sigmoid(linear(h, w[p + "b"]))
    g = np.exp(-np.exp(array(w[p + "A_log"])) * softplus(linear(h, w[p + "a"]) + array(w[p + "dt_bias"])))
    o, _ = delta_scan(unit(q) * d ** -0.5, unit(k), v, beta, g)
    o = rms_norm(o, w[p + "norm"], eps).reshape(t_len, heads * dv)
    return linear(o * silu(linear(h, w[p + "g"])), w[p + "o"])


# ----------------------------------------------------------------------------- feed-forward

def dense_ff(w, p, h):
    return linear(np.maximum(linear(h, w[p + "up"]), 0.0) ** 2, w[p + "down"])


def expert_ff(w, p, h):
    return linear(silu(linear(h, w[p + "gate"])) * linear(h, w[p + "up"]), w[p + "down"])


def route(z, correction, top, group_count=1, group_keep=1):
    """z [experts] router logits of one token -> (chosen experts, their weights, the margin of the choice)."""
    z = array(z)
    e = np.exp(z - z.max())
    s = e / e.sum()
    c = s + array(correction)
    size = len(s) // group_count
    group_score = np.array([c[g * size:(g + 1) * size].max() for g in range(group_count)])
    order = sorted(range(group_count), key=lambda g: (-group_score[g], g))
    kept = set(order[:group_keep])
    open_to = [x for x in range(len(s)) if x // size in kept]
    ranked = sorted(open_to, key=lambda x: (-c[x], x))
    chosen = ranked[:top]
    weights = s[chosen] / (s[chosen].sum() + ROUTE_EPS)
    margin = c[ranked[top - 1]] - c[ranked[top]] if top < len(ranked) else np.inf
    if group_keep < group_count:
        margin = min(margin, group_score[order[group_keep - 1]] - group_score[order[group_keep]])
    return chosen, weights, margin


def routed_ff(w, p, mlp, h, margins=None):
    r = mlp["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    z = linear(h, w[p + "router"])
    assert z.shape[1] == r["experts"] + (r.get("identity") or 0)
    out = np.zeros_like(array(h))
    for t in range(h.shape[0]):
        chosen, weights, margin = route(z[t], w[p + "correction"], r["top"], groups["count"], groups["keep"])
        if margins is not None:
            margins.append(margin)
        for e, weight in zip(chosen, weights):
            out[t] += weight * (expert_ff(w, f"{p}e{e}.", h[t:t + 1])[0] if e < r["experts"] else h[t])
    if mlp.get("shared") is not None:
        out += sigmoid(linear(h, w[p + "shared.sg"])) * expert_ff(w, p + "shared.", h)
    return out


MIXERS = {"rglru": recurrent_mixer, "parallel": parallel_mixer, "delta": delta_mixer}


def forward_whole(cfg, w, tokens, layers_out=None, margins=None):
    """Logits [T, vocab] of a whole sequence.  `layers_out`: a list that receives X after every layer run."""
    eps = cfg["norm"]["eps"]
    x = array(w["embed"])[list(tokens)] * cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{layer['weights_of'] if layer.get('weights_of') is not None else i}."
        x = x + MIXERS[layer["type"]](w, p + "mix.", layer["mixer"], rms_norm(x, w[p + "norm1"], eps), eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            h = rms_norm(x, w[p + "norm2"], eps)
            x = x + (dense_ff(w, p + "mlp.", h) if mlp["kind"] == "dense" else routed_ff(w, p + "mlp.", mlp, h, margins))
        if layers_out is not None:
            layers_out.append(x.copy())
    return linear(rms_norm(x, w["final.norm"], eps), w["head"])


def load_folder(folder):
    """(config dict, {name: float64 array}) of a model folder."""
    import torch
    from safetensors.torch import load_file
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    tensors = load_file(os.path.join(folder, "model.safetensors"))
    return cfg, {k: v.to(torch.float64).numpy() for k, v in tensors.items()}
