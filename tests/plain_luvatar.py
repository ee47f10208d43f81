"""A plain, slow Luvatar in NumPy float64: one function per mechanism, whole sequences only, no cache and no
state kept between calls.  It is what the engine is compared with; it shares no code with it (the model folder
is read with the safetensors package, the formulas are written out here).

``r`` is applied to what a 16-bit engine rounds (inputs of matrix products, projections, keys and values as a cache holds
them, the heads' gated results): the identity as a rule; with a rounding function the difference to the unrounded result
says how far rounding alone moves a position's logits in a given model."""
from __future__ import annotations

import json
import os

import numpy as np


def exact(x):
    return x


def read_model_folder(folder):
    """config.json as a dict, tensors as float64 NumPy arrays by name."""
    import torch
    from safetensors import safe_open
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    tensors = {}
    with safe_open(os.path.join(folder, "model.safetensors"), framework="pt") as f:
        for name in f.keys():
            tensors[name] = f.get_tensor(name).to(torch.float64).numpy()
    return cfg, tensors


# --------------------------------------------------------------------------- small functions
def rms_scaled(x, gain, eps):
    """Rows divided by their root mean square (eps under the root), times a gain."""
    return x / np.sqrt(np.mean(np.square(x), axis=-1, keepdims=True) + eps) * gain


def logistic(z):
    return 1.0 / (1.0 + np.exp(-z))


def swish(z):
    return z * logistic(z)


def log_logistic(z):
    """ln logistic(z), also far below zero."""
    return -np.logaddexp(0.0, -z)


# --------------------------------------------------------------------------- positions
def pair_speeds(rot):
    """Speed of every pair: base^(-2i / dims), all divided by the scaling's factor when there is one."""
    dims = rot["dims"]
    speeds = np.array([float(rot["base"]) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=np.float64)
    scaling = rot.get("scaling")
    return speeds / float(scaling["factor"]) if scaling else speeds


def turn_neighbours(v, places, rot):
    """v [T, ..., d]: entries 2i and 2i + 1 among the first ``dims`` are turned by the angle place * speed_i; what
    lies behind passes."""
    if rot is None or not rot["dims"]:
        return v.copy()
    dims = rot["dims"]
    out = v.copy()
    ang = np.asarray(places, dtype=np.float64)[:, None] * pair_speeds(rot)[None, :]
    shape = (len(places),) + (1,) * (v.ndim - 2) + (dims // 2,)
    c, s = np.cos(ang).reshape(shape), np.sin(ang).reshape(shape)
    a, b = v[..., 0:dims:2], v[..., 1:dims:2]
    out[..., 0:dims:2] = a * c - b * s
    out[..., 1:dims:2] = b * c + a * s
    return out


def chunk_mask(T, size):
    """[T, T] True where row i sees column j: j <= i in the same chunk of ``size`` positions (None: every j <= i)."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) if size is None else (j <= i) & (i // size == j // size)


def softmax_with_sink(scores, mask, sink):
    """Rows of weights exp(s_j) / (exp(sink) + sum over seen j of exp(s_j))."""
    s = np.where(mask, scores, -np.inf)
    m = np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.where(mask, np.exp(s - m), 0.0)
    return e / (np.exp(sink - m) + e.sum(axis=-1, keepdims=True))


# --------------------------------------------------------------------------- mixers
def keys_and_values(W, p, m, h, eps, r=exact):
    """(keys [T, G, dim] normalised and turned, values [T, G, vdim]) of an attention layer with projections of its own."""
    T, G = h.shape[0], m["kv_heads"]
    k = (h @ W[p + "mix.k"].T).reshape(T, G, m["dim"])
    k = turn_neighbours(rms_scaled(k, W[p + "mix.k.norm"], eps), np.arange(T), m["rot"])
    return r(k), r((h @ W[p + "mix.v"].T).reshape(T, G, m["vdim"]))


def attention(W, p, m, h, eps, kv, r=exact):
    """Softmax attention inside chunks with grouped key heads, a norm of each head's query, one more learned term in
    the denominator, and a logistic gate of the input on the heads' results.  ``kv``: keys and values, the layer's own
    or another layer's."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    k, v = kv
    q = rms_scaled((h @ W[p + "mix.q"].T).reshape(T, H, m["dim"]), W[p + "mix.q.norm"], eps)
    q = r(turn_neighbours(q, np.arange(T), m["rot"]))
    mask = chunk_mask(T, (m.get("mask") or {}).get("size"))
    out = np.zeros((T, H, m["vdim"]))
    for hd in range(H):
        g = hd // (H // G)
        w = softmax_with_sink((q[:, hd] @ k[:, g].T) * m["scale"], mask, W[p + "mix.sink"][hd])
        out[:, hd] = w @ v[:, g]
    return r(out.reshape(T, -1) * logistic(r(h @ W[p + "mix.g"].T))) @ W[p + "mix.o"].T


def gated_linear(W, p, m, h, eps, r=exact):
    """Per head S <- diag(alpha) S + k v^T, o = S^T q, token by token from S = 0, with a decay alpha per key channel,
    alpha = logistic(z)^(1 / tau), z a low-rank projection plus a bias; o is normalised per head, gated by swish of a
    projection, and projected back."""
    T, H, D, Dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = r(h @ W[p + "mix.q"].T).reshape(T, H, D) * D ** -0.5
    k = r(h @ W[p + "mix.k"].T).reshape(T, H, D)
    v = r(h @ W[p + "mix.v"].T).reshape(T, H, Dv)
    z = r(h @ W[p + "mix.a1"].T) @ W[p + "mix.a2"].T + W[p + "mix.a2.b"]
    alpha = np.exp(log_logistic(z) / m["tau"]).reshape(T, H, D)
    S = np.zeros((H, D, Dv))
    o = np.zeros((T, H, Dv))
    for t in range(T):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    o = rms_scaled(o, W[p + "mix.norm"], eps).reshape(T, H * Dv)
    return r(o * swish(r(h @ W[p + "mix.g"].T))) @ W[p + "mix.o"].T


def feed_forward(W, p, h, r=exact):
    return r(swish(r(h @ W[p + "gate"].T)) * r(h @ W[p + "up"].T)) @ W[p + "down"].T


# --------------------------------------------------------------------------- the model
def forward(cfg, W, ids, layers_out=None, r=exact):
    """Logits [T, V] of one whole sequence.  ``layers_out``: a list that receives the stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][np.asarray(ids)] * cfg["embedding"]["scale"]
    kept = {}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        if L["type"] == "gla":
            y = gated_linear(W, p, m, r(x), eps, r)
        elif L["type"] == "attention":
            src = m.get("kv_from")
            kept[i] = kept[src] if src is not None else keys_and_values(W, p, m, r(x), eps, r)
            y = attention(W, p, m, r(x), eps, kept[i], r)
        else:
            raise ValueError(L["type"])
        x = x + rms_scaled(y, W[p + "norm1"], eps)
        if L.get("mlp"):
            x = x + rms_scaled(feed_forward(W, p + "mlp.", r(x), r), W[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return r(rms_scaled(x, W["final.norm"], eps)) @ W["embed"].T


def forward_logits(cfg, W, ids):
    return forward(cfg, W, ids)


def greedy_generate(cfg, W, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(np.argmax(forward(cfg, W, ids)[-1])))
    return ids[len(prompt):]
