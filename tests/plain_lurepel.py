"""A plain, slow implementation of the Lurepel decoder in NumPy: whole sequences, no cache, no batches, one function per
mechanism, float64 sums.  It shares no code with the package and is the oracle of the tests.

The design in this file's notation (T tokens, width D, n(x; w) = x / sqrt(mean(x^2) + eps) * w, u(x) the same without w):
  embedding      x = n(E[token]; w_embed)
  layer          x <- x + n(M(x); w1);  x <- x + n(F(x); w2)   (F may be absent): only what a sublayer gives is normed
  mixer M        q_h = u(R_p (Wq x)_h),  k_g = u(R_p (Wk x)_g),  v_g = (Wk x)_g: a value is its own key before turn and norm
                 s_ij = (q_i . k_j) * scale  for j <= i with i and j in the same chunk (floor(i / size) = floor(j / size));
                 p_ij = exp(s_ij) / (1 + sum_j exp(s_ij));  o_h = sigmoid(Wg x)_h sum_j p_ij v_j;  M(x) = Wo concat_h o_h
  rotation R_p   neighbours (2i, 2i+1) of the first `dims` dimensions of a head turned by p * f_i, f_i = base^(-2i/dims), slow
                 pairs slowed further by wavelength (below)
  dense F        Wdown (gelu(Wgate x) * (Wup x)), gelu in its tanh form
  experts F      s = softmax(Wr x) over all of them; the `top` with the largest s + correction; sum of s_e E_e(x), the shares as
                 they are; E_e(x) = Wd (silu(Wg x) * (Wu x)), the last `identity` of the experts are E(x) = x
  output         logits = H n(x; w_final)
"""

from __future__ import annotations

import json
import math
import os

import numpy as np

F64 = np.float64


def load(folder):
    """(config dictionary, {name: float32 array}) of a model folder."""
    import torch
    from safetensors import safe_open

    with open(os.path.join(folder, "config.json")) as handle:
        config = json.load(handle)
    with safe_open(os.path.join(folder, "model.safetensors"), framework="pt") as handle:
        weights = {name: handle.get_tensor(name).to(torch.float32).numpy() for name in handle.keys()}
    return config, weights


def f64(a):
    return np.asarray(a, F64)


def linear(x, w):
    return f64(x) @ f64(w).T


def unit(x, eps):
    """x over its root mean square."""
    x = f64(x)
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def norm(x, w, eps):
    return unit(x, eps) * f64(w)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-f64(z)))


def silu(z):
    return f64(z) * sigmoid(z)


def gelu(z):
    z = f64(z)
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def frequencies(rot):
    """The turn per position of every pair of a rotation block {base, dims, scaling?}.  With `scaling` a pair whose wave is
    longer than original / low positions turns `factor` times slower, one shorter than original / high as it is, and in
    between the two are mixed by how many waves fit into `original` positions."""
    dims = int(rot["dims"])
    plain = float(rot["base"]) ** (-2.0 * np.arange(dims // 2, dtype=F64) / dims)
    scaling = rot.get("scaling")
    if not scaling:
        return plain
    factor, low, high, original = (float(scaling[key]) for key in ("factor", "low", "high", "original"))
    out = []
    for f in plain:
        wave = 2.0 * math.pi / f
        if wave < original / high:
            out.append(f)
        elif wave > original / low:
            out.append(f / factor)
        else:
            share = (original / wave - low) / (high - low)
            out.append((1.0 - share) * f / factor + share * f)
    return np.array(out, F64)


def turn(x, positions, rot):
    """x [T, heads, dim]: dimensions 2i and 2i + 1 (i < dims / 2) of every head turned by position * f_i; the rest passes."""
    dims = int(rot["dims"])
    angles = f64(positions)[:, None, None] * frequencies(rot)[None, None, :]
    out = f64(x).copy()
    a, b = out[..., 0:dims:2].copy(), out[..., 1:dims:2].copy()
    out[..., 0:dims:2] = a * np.cos(angles) - b * np.sin(angles)
    out[..., 1:dims:2] = b * np.cos(angles) + a * np.sin(angles)
    return out


def seen(t_len, chunk, first_position=0):
    """[query, key] booleans: keys up to the query's own, within its chunk of positions (0: every earlier one)."""
    at = first_position + np.arange(t_len)
    visible = at[None, :] <= at[:, None]
    if chunk:
        visible &= (at[None, :] // chunk) == (at[:, None] // chunk)
    return visible


def softmax_with_one_more(scores, visible):
    """exp(s) / (1 + sum exp(s)) over the visible keys of every row."""
    masked = np.where(visible, scores, -np.inf)
    top = np.maximum(masked.max(axis=-1, keepdims=True), 0.0)
    e = np.where(visible, np.exp(masked - top), 0.0)
    return e / (np.exp(-top) + e.sum(axis=-1, keepdims=True))


def attend(q, k, v, scale, visible):
    """q [T, H, d], k [S, G, d], v [S, G, d]; query head h reads key/value head h // (H / G)."""
    heads, per = q.shape[1], q.shape[1] // k.shape[1]
    out = np.zeros((q.shape[0], heads, v.shape[2]), F64)
    for h in range(heads):
        scores = f64(q[:, h]) @ f64(k[:, h // per]).T * scale
        out[:, h] = softmax_with_one_more(scores, visible) @ f64(v[:, h // per])
    return out


def attention(h, w, p, m, eps, first_position=0):
    t_len = h.shape[0]
    heads, groups, dim = m["heads"], m["kv_heads"], m["dim"]
    positions = first_position + np.arange(t_len)
    q = linear(h, w[p + "q"]).reshape(t_len, heads, dim)
    k = linear(h, w[p + "k"]).reshape(t_len, groups, dim)
    v = k
    if m.get("rot"):
        q, k = turn(q, positions, m["rot"]), turn(k, positions, m["rot"])
    q, k = unit(q, eps), unit(k, eps)
    chunk = int(m["mask"]["size"]) if m.get("mask") else 0
    out = attend(q, k, v, float(m["scale"]), seen(t_len, chunk, first_position))
    out = out * sigmoid(linear(h, w[p + "g"]))[:, :, None]
    return linear(out.reshape(t_len, heads * dim), w[p + "o"])


def dense(h, w, p):
    return linear(gelu(linear(h, w[p + "gate"])) * linear(h, w[p + "up"]), w[p + "down"])


def expert(h, w, p):
    return linear(silu(linear(h, w[p + "gate"])) * linear(h, w[p + "up"]), w[p + "down"])


def softmax(z):
    e = np.exp(z - z.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def route(h, w, p, top):
    """-> (chosen [T, top] by falling choice score, ties to the lower index; their shares of the softmax over all)."""
    shares = softmax(linear(h, w[p + "router"]))
    choice = shares + f64(w[p + "correction"])
    chosen = np.argsort(-choice, axis=-1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(shares, chosen, axis=-1)


def experts(h, w, p, mlp):
    router = mlp["router"]
    chosen, shares = route(h, w, p, int(router["top"]))
    out = np.zeros_like(f64(h))
    for e in range(int(router["experts"]) + int(router.get("identity", 0))):
        share = np.where(chosen == e, shares, 0.0).sum(axis=-1)
        rows = np.nonzero((chosen == e).any(axis=-1))[0]
        if len(rows):
            given = f64(h)[rows] if e >= int(router["experts"]) else expert(f64(h)[rows], w, f"{p}e{e}.")
            out[rows] += share[rows, None] * given
    return out


def feed_forward(h, w, p, mlp):
    return dense(h, w, p) if mlp["kind"] == "dense" else experts(h, w, p, mlp)


def forward(config, w, tokens, residuals=None):
    """Logits [T, vocab] (float64) of a whole sequence; `residuals`: a list that gets x after every layer."""
    eps = float(config["norm"]["eps"])
    x = norm(f64(w["embed"])[np.asarray(tokens)], w["embed.norm"], eps)
    for index, layer in enumerate(config["layers"]):
        p = f"l{index}."
        x = x + norm(attention(x, w, p + "mix.", layer["mixer"], eps), w[p + "norm1"], eps)
        if layer.get("mlp"):
            x = x + norm(feed_forward(x, w, p + "mlp.", layer["mlp"]), w[p + "norm2"], eps)
        if residuals is not None:
            residuals.append(x.copy())
    return linear(norm(x, w["final.norm"], eps), w["head"])


def greedy(config, w, prompt, n_new):
    """The tokens that greedy decoding appends (ties to the lowest id), each from a whole forward of what stands so far."""
    tokens = list(prompt)
    for _ in range(n_new):
        tokens.append(int(np.argmax(forward(config, w, tokens)[-1])))
    return tokens[len(prompt):]
