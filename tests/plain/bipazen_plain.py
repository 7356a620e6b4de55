"""The plain implementation of the Bipazen decoder: whole sequences, no cache, no pages, no batching, one function for
each mechanism, NumPy float64.  It shares no code with `kipp_amd`; model folders are read with the `safetensors` package.

Notation: a sequence has T tokens at positions 0 .. T-1, X [T, width] is the residual stream, N(x; w) = x / sqrt(mean
x^2 + eps) * w.

    input            X = embed[tokens]
    layer            X += ls1 * mixer(N(X; norm1));  X += ls2 * ff(N(X; norm2))     (element by element; a layer may have no ff;
                     a layer may name another whose tensors it uses)
    mamba2           [z | x | B | C | dt] = W_in h;  x, B, C through a causal filter a channel (with bias) and silu;
                     dt = softplus(dt + dt_bias);  S_t = exp(-exp(A_h) dt) S_(t-1) + dt B_t x_t^T;  y_t = S_t^T C_t + D_h x_t;
                     y * silu(z), then N in `norm_groups` equal parts (times .norm), then Wo
    rglru            y = gelu_tanh(Wy h + by);  u = filter(Wx h + bx) + b;  in every block of u: r = sigmoid(Ra u + ba),
                     i = sigmoid(Ri u + bi);  log a = -8 r softplus(lam);  S_t = a S_(t-1) + sqrt(1 - a^2) i u;  Wo (S * y)
    latent attention q = Wq h, a head [dim | rot_dim];  [c' | kr] = Wdkv h, c = N(c'; dkv.norm);  a head's key [Wuk c | kr], its
                     value Wuv c;  the rot_dim parts turned by the position (halves paired);  softmax over every earlier
                     position of scale q . k;  the heads side by side times sigmoid(Wg h), then Wo
    experts          s = sigmoid(Wr h); the `top` largest are chosen; sum over them of E_e(s_e h),
                     E(u) = Wdown (silu(Wgate u) * Wup u)
    output           logits = embed N(X; final.norm)
"""
from __future__ import annotations

import json
import math
import os

import numpy as np

DTYPE = np.float64
RECURRENCE_FACTOR = 8.0


def linear(x, w, b=None):
    y = np.asarray(x, dtype=DTYPE) @ np.asarray(w, dtype=DTYPE).T
    return y if b is None else y + np.asarray(b, dtype=DTYPE)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return np.logaddexp(0.0, z)


def rms_norm(x, w, eps):
    x = np.asarray(x, dtype=DTYPE)
    y = x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)
    return y if w is None else y * np.asarray(w, dtype=DTYPE)


def causal_filter(x, taps_w, bias, before=None):
    """x [T, C], taps_w [C, taps] (the last column weighs the current token's input), zeros (or `before`
    [taps - 1, C]) ahead of the first token."""
    x = np.asarray(x, dtype=DTYPE)
    taps_w = np.asarray(taps_w, dtype=DTYPE)
    taps = taps_w.shape[1]
    ahead = np.zeros((taps - 1, x.shape[1]), dtype=DTYPE) if before is None else np.asarray(before, dtype=DTYPE)
    full = np.concatenate([ahead, x], axis=0)
    out = np.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(taps):
            out[t] += taps_w[:, j] * full[t + j]
    return out + np.asarray(bias, dtype=DTYPE)


def state_space_scan(x, b, c, dt, a_log, d_skip, state=None):
    """x [T, H, P], b and c [T, G, N], dt [T, H] (after softplus): S_t = exp(-exp(A_h) dt) S_(t-1) + dt B_t x_t^T,
    y_t = S_t^T C_t + D_h x_t.  Returns (y [T, H, P], S [H, N, P])."""
    t_len, heads, p = x.shape
    groups, n = b.shape[1], b.shape[2]
    rep = heads // groups
    s = np.zeros((heads, n, p), dtype=DTYPE) if state is None else np.array(state, dtype=DTYPE)
    y = np.zeros((t_len, heads, p), dtype=DTYPE)
    for t in range(t_len):
        for h in range(heads):
            g = h // rep
            s[h] = math.exp(-math.exp(a_log[h]) * dt[t, h]) * s[h] + dt[t, h] * np.outer(b[t, g], x[t, h])
            y[t, h] = s[h].T @ c[t, g] + d_skip[h] * x[t, h]
    return y, s


def state_space_mixer(w, prefix, m, h, eps):
    t_len = h.shape[0]
    heads, p, n, groups = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = heads * p
    proj = linear(h, w[prefix + "in"])
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * groups * n], proj[:, 2 * inner + 2 * groups * n:]
    assert dt.shape[1] == heads
    xbc = silu(causal_filter(xbc, w[prefix + "conv"], w[prefix + "conv.b"]))
    x = xbc[:, :inner].reshape(t_len, heads, p)
    b = xbc[:, inner:inner + groups * n].reshape(t_len, groups, n)
    c = xbc[:, inner + groups * n:].reshape(t_len, groups, n)
    dt = softplus(dt + np.asarray(w[prefix + "dt_bias"], dtype=DTYPE))
    y, _ = state_space_scan(x, b, c, dt, np.asarray(w[prefix + "A_log"], dtype=DTYPE), np.asarray(w[prefix + "D"], dtype=DTYPE))
    y = y.reshape(t_len, inner) * silu(z)
    parts = m["norm_groups"]
    y = rms_norm(y.reshape(t_len, parts, inner // parts), None, eps).reshape(t_len, inner) * np.asarray(w[prefix + "norm"], dtype=DTYPE)
    return linear(y, w[prefix + "o"])


def block_gates(u, ra, ra_b, ri, ri_b):
    """u [T, width] in len(ra) equal blocks -> (r, i) [T, width]: sigmoid of a square matrix of each block's own, with a bias."""
    t_len, width = u.shape
    blocks = len(ra)
    size = width // blocks
    r, i = np.zeros_like(u), np.zeros_like(u)
    for b in range(blocks):
        part = slice(b * size, (b + 1) * size)
        r[:, part] = sigmoid(linear(u[:, part], ra[b], ra_b[b]))
        i[:, part] = sigmoid(linear(u[:, part], ri[b], ri_b[b]))
    return r, i


def gated_recurrence(u, r, i, lam, state=None):
    """log a = -8 r softplus(lam); S_t = a_t S_(t-1) + sqrt(1 - a_t^2) i_t u_t, channel by channel.  Returns (S of every token, the last S)."""
    log_a = -RECURRENCE_FACTOR * r * softplus(np.asarray(lam, dtype=DTYPE))
    a = np.exp(log_a)
    x = np.sqrt(-np.expm1(2.0 * log_a)) * i * u
    s = np.zeros(u.shape[1], dtype=DTYPE) if state is None else np.array(state, dtype=DTYPE)
    out = np.zeros_like(u)
    for t in range(u.shape[0]):
        s = a[t] * s + x[t]
        out[t] = s
    return out, s


def recurrent_mixer(w, prefix, m, h):
    y = gelu_tanh(linear(h, w[prefix + "y"], w[prefix + "y.b"]))
    u = causal_filter(linear(h, w[prefix + "x"], w[prefix + "x.b"]), w[prefix + "conv"], w[prefix + "conv.b"])
    assert u.shape[1] == m["width"] and w[prefix + "conv"].shape[1] == m["conv"] and len(w[prefix + "ra"]) == m["blocks"]
    r, i = block_gates(u, w[prefix + "ra"], w[prefix + "ra.b"], w[prefix + "ri"], w[prefix + "ri.b"])
    s, _ = gated_recurrence(u, r, i, w[prefix + "lam"])
    return linear(s * y, w[prefix + "o"])


def rotate(x, positions, dims, base):
    """x [T, heads, d]: the first `dims` numbers of every head turned, number i paired with number i + dims / 2."""
    x = np.array(x, dtype=DTYPE)
    half = dims // 2
    freq = np.array([float(base) ** (-2.0 * i / dims) for i in range(half)], dtype=DTYPE)
    angle = np.asarray(positions, dtype=DTYPE)[:, None] * freq[None, :]
    cos, sin = np.cos(angle)[:, None, :], np.sin(angle)[:, None, :]
    u, v = x[..., :half].copy(), x[..., half:dims].copy()
    x[..., :half] = u * cos - v * sin
    x[..., half:dims] = v * cos + u * sin
    return x


def causal_attention(q, k, v, scale):
    """q, k [T, H, d], v [T, H, dv]: softmax over j <= i."""
    out = np.zeros((q.shape[0], q.shape[1], v.shape[2]), dtype=DTYPE)
    for i in range(q.shape[0]):
        s = np.einsum("hd,jhd->hj", q[i], k[:i + 1]) * scale
        e = np.exp(s - s.max(axis=1, keepdims=True))
        out[i] = np.einsum("hj,jhd->hd", e / e.sum(axis=1, keepdims=True), v[:i + 1])
    return out


def latent_attention(w, prefix, m, h, positions, eps):
    t_len = h.shape[0]
    heads, d, dr, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = linear(h, w[prefix + "q"]).reshape(t_len, heads, d + dr)
    down = linear(h, w[prefix + "dkv"])
    c, kr = rms_norm(down[:, :rank], w[prefix + "dkv.norm"], eps), down[:, rank:].reshape(t_len, 1, dr)
    k = linear(c, w[prefix + "uk"]).reshape(t_len, heads, d)
    v = linear(c, w[prefix + "uv"]).reshape(t_len, heads, dv)
    qr = q[..., d:]
    if dr:
        rot = m["rot"]
        qr, kr = rotate(qr, positions, rot["dims"], rot["base"]), rotate(kr, positions, rot["dims"], rot["base"])
    q = np.concatenate([q[..., :d], qr], axis=-1)
    k = np.concatenate([k, np.repeat(kr, heads, axis=1)], axis=-1)
    o = causal_attention(q, k, v, m["scale"]).reshape(t_len, heads * dv)
    return linear(o * sigmoid(linear(h, w[prefix + "g"])), w[prefix + "o"])


def route(z, top):
    """z [E] router logits of one token -> (chosen experts, their weights, the margin of the choice)."""
    s = sigmoid(np.asarray(z, dtype=DTYPE))
    ranked = sorted(range(len(s)), key=lambda e: (-s[e], e))
    chosen = ranked[:top]
    margin = s[ranked[top - 1]] - s[ranked[top]] if top < len(s) else np.inf
    return chosen, s[chosen], margin


def expert(w, prefix, u):
    return linear(silu(linear(u, w[prefix + "gate"])) * linear(u, w[prefix + "up"]), w[prefix + "down"])


def routed_ff(w, prefix, mlp, h, margins=None):
    z = linear(h, w[prefix + "router"])
    assert z.shape[1] == mlp["router"]["experts"]
    out = np.zeros_like(h, dtype=DTYPE)
    for t in range(h.shape[0]):
        chosen, weights, margin = route(z[t], mlp["router"]["top"])
        if margins is not None:
            margins.append(margin)
        for e, wt in zip(chosen, weights):
            out[t] += expert(w, f"{prefix}e{e}.", wt * h[t:t + 1])[0]
    return out


def owner_of(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward_whole(cfg, w, tokens, layers_out=None, margins=None):
    """Logits [T, vocab] of a whole sequence.  `layers_out`: a list that receives X after every layer."""
    eps = cfg["norm"]["eps"]
    positions = list(range(len(tokens)))
    x = np.asarray(w["embed"], dtype=DTYPE)[list(tokens)]
    for i, layer in enumerate(cfg["layers"]):
        at = f"l{owner_of(cfg, i)}."
        h = rms_norm(x, w[at + "norm1"], eps)
        m, kind = layer["mixer"], layer["type"]
        if kind == "mamba2":
            delta = state_space_mixer(w, at + "mix.", m, h, eps)
        elif kind == "rglru":
            delta = recurrent_mixer(w, at + "mix.", m, h)
        elif kind == "latent_attention":
            delta = latent_attention(w, at + "mix.", m, h, positions, eps)
        else:
            raise ValueError(f"layer type {kind!r}")
        x = x + np.asarray(w[at + "ls1"], dtype=DTYPE) * delta
        mlp = layer.get("mlp")
        if mlp is not None:
            if mlp["kind"] != "moe":
                raise ValueError(f"feed-forward kind {mlp['kind']!r}")
            h = rms_norm(x, w[at + "norm2"], eps)
            x = x + np.asarray(w[at + "ls2"], dtype=DTYPE) * routed_ff(w, at + "mlp.", mlp, h, margins)
        if layers_out is not None:
            layers_out.append(x.copy())
    return linear(rms_norm(x, w["final.norm"], eps), w["embed"])


def load_folder(folder):
    """(config dict, {name: float64 array}) of a model folder."""
    import torch
    from safetensors.torch import load_file
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    tensors = load_file(os.path.join(folder, "model.safetensors"))
    return cfg, {k: v.to(torch.float64).numpy() for k, v in tensors.items()}
