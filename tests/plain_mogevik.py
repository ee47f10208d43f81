"""A plain, slow Mogevik in NumPy float64: one function per mechanism, whole sequences only, no cache and no state kept
between calls.  It is what the engine is compared with; it shares no code with it (the model folder is read with the
safetensors package, the formulas are written out here).

``r`` is applied to what a 16-bit engine rounds (norm outputs that enter matrix products, projections, filtered inputs,
keys and values as a cache holds them, the mixers' gated results, the experts' middles): the identity as a rule; with a
rounding function the difference to the unrounded result says how far rounding alone moves a position's logits."""
from __future__ import annotations

import json
import math
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
def layer_norm(x, gain, eps):
    """Rows with their mean taken off, divided by the root of their mean squared deviation plus eps, times a gain."""
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt((d * d).mean(axis=-1, keepdims=True) + eps) * gain


def logistic(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def swish(z):
    return z * logistic(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return np.logaddexp(0.0, z)


# --------------------------------------------------------------------------- the recurrent mixer
def causal_filter(x, taps, bias):
    """x [T, C], taps [C, K]: y[t, c] = bias[c] + sum_k taps[c, k] x[t - (K - 1 - k), c]; nothing before the start."""
    T, K = x.shape[0], taps.shape[1]
    y = np.tile(bias, (T, 1)).astype(np.float64)
    for k in range(K):
        back = K - 1 - k
        if back < T:
            y[back:] += taps[:, k] * x[:T - back]
    return y


def per_block(u, mats, bias):
    """u [T, C] in len(mats) equal parts; part b goes through the square matrix mats[b] [out, in] and bias[b]."""
    T, (B, n, _) = u.shape[0], mats.shape
    parts = u.reshape(T, B, n)
    return np.stack([parts[:, b] @ mats[b].T + bias[b] for b in range(B)], axis=1).reshape(T, B * n)


def gated_walk(u, decay_logit, input_logit, lam, strength=8.0):
    """S_t = a_t S_(t-1) + sqrt(1 - a_t^2) logistic(input_logit) u_t channel by channel from S = 0, with
    a = exp(-strength * logistic(decay_logit) * softplus(lam)); every S [T, C]."""
    log_a = -strength * logistic(decay_logit) * softplus(lam)
    add = np.sqrt(-np.expm1(2.0 * log_a)) * logistic(input_logit) * u
    S, out = np.zeros(u.shape[1]), np.zeros_like(u)
    for t in range(len(u)):
        S = np.exp(log_a[t]) * S + add[t]
        out[t] = S
    return out


def recurrent_block(W, p, h, r=exact):
    y = gelu_tanh(r(h @ W[p + "mix.y"].T + W[p + "mix.y.b"]))
    u = r(causal_filter(r(h @ W[p + "mix.x"].T + W[p + "mix.x.b"]), W[p + "mix.conv"], W[p + "mix.conv.b"]))
    S = gated_walk(u, per_block(u, W[p + "mix.ra"], W[p + "mix.ra.b"]), per_block(u, W[p + "mix.ri"], W[p + "mix.ri.b"]),
                   W[p + "mix.lam"])
    return r(S * y) @ W[p + "mix.o"].T


# --------------------------------------------------------------------------- attention
def head_slopes(H):
    return np.array([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)])


def seen(T, window):
    """[T, T] True where row i sees column j: the window's last ``window`` positions, itself among them."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) if window is None else (j <= i) & (i - j < window)


def softmax_rows(scores, mask):
    s = np.where(mask, scores, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def attention(W, p, m, h, r=exact):
    """Softmax attention over a window with grouped key heads; a score loses its head's slope for every position of
    distance; a logistic gate of the input multiplies the heads' results."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = r(h @ W[p + "mix.q"].T + W[p + "mix.q.b"]).reshape(T, H, m["dim"])
    k = r(h @ W[p + "mix.k"].T + W[p + "mix.k.b"]).reshape(T, G, m["dim"])
    v = r(h @ W[p + "mix.v"].T + W[p + "mix.v.b"]).reshape(T, G, m["vdim"])
    far = np.arange(T)[:, None] - np.arange(T)[None, :]
    mask, slopes = seen(T, (m.get("mask") or {}).get("size")), head_slopes(H)
    out = np.zeros((T, H, m["vdim"]))
    for hd in range(H):
        g = hd // (H // G)
        out[:, hd] = softmax_rows((q[:, hd] @ k[:, g].T) * m["scale"] - slopes[hd] * far, mask) @ v[:, g]
    return r(out.reshape(T, -1) * logistic(r(h @ W[p + "mix.g"].T))) @ W[p + "mix.o"].T


# --------------------------------------------------------------------------- experts
def expert(W, p, h, r=exact):
    return r(swish(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def softmax(z):
    e = np.exp(z - z.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def choose(z, correction, top, groups=None):
    """Router logits z [T, n] -> (chosen [T, top], weights [T, top]).  The softmax over all of them plus the correction
    decides; with groups, only entries of the best ``keep`` of ``count`` runs of neighbours (a run counts as its largest
    entry) can be chosen.  The weights are the chosen softmax scores without the correction, over their sum."""
    T, n = z.shape
    s = softmax(z)
    c = s + correction
    if groups:
        count, keep = groups["count"], groups["keep"]
        runs = c.reshape(T, count, n // count)
        best = np.argsort(-runs.max(axis=2), axis=1, kind="stable")[:, :keep]
        open_ = np.zeros((T, count), dtype=bool)
        np.put_along_axis(open_, best, True, axis=1)
        c = np.where(open_[:, :, None], runs, -np.inf).reshape(T, n)
    chosen = np.argsort(-c, axis=1, kind="stable")[:, :top]
    return chosen, weights_of(s, chosen)


def weights_of(s, chosen):
    w = np.take_along_axis(s, chosen, axis=1)
    return w / (w.sum(axis=1, keepdims=True) + 1e-20)


def nearly_as_good(c, theirs, groups, slack):
    """Whether the entries ``theirs`` are a choice from c [n] that an error of ``slack`` in the scores would explain."""
    if len(set(theirs)) != len(theirs):
        return False
    open_ = np.ones(len(c), dtype=bool)
    if groups:
        count, keep = groups["count"], groups["keep"]
        size = len(c) // count
        top_of = c.reshape(count, size).max(axis=1)
        used = {e // size for e in theirs}
        order = np.argsort(-top_of, kind="stable")
        if len(used) > keep or any(top_of[g] < top_of[order[keep - 1]] - slack for g in used):
            return False
        for g in order:                                # the groups that are left to be kept are the best of the rest
            if len(used) < keep:
                used.add(int(g))
        open_ = np.isin(np.arange(len(c)) // size, sorted(used))
    floor = np.sort(c[open_])[-len(theirs)]
    return all(c[e] >= floor - slack for e in theirs)


def experts(W, p, mlp, h, r=exact, routes=None, slack=0.0):
    """``routes`` (position -> entries chosen elsewhere): followed where they are as good as the own choice within
    ``slack`` of choice score, with the weights that go with them."""
    ro = mlp["router"]
    n = ro["experts"]
    z = h @ W[p + "router"].T
    chosen, w = choose(z, W[p + "correction"], ro["top"], ro.get("groups"))
    if routes is not None:
        s = softmax(z)
        for t in range(len(h)):
            if t in routes and sorted(routes[t]) != sorted(chosen[t].tolist()) and \
                    nearly_as_good(s[t] + W[p + "correction"], routes[t], ro.get("groups"), slack):
                chosen[t] = routes[t]
        w = weights_of(s, chosen)
    out = np.zeros_like(h)
    for e in range(n + (ro.get("identity") or 0)):
        t, k = np.nonzero(chosen == e)
        if len(t):
            y = expert(W, f"{p}e{e}.", h[t], r) if e < n else h[t]
            out[t] += w[t, k][:, None] * y
    if mlp.get("shared"):
        out = out + logistic(h @ W[p + "shared.sg"].T) * expert(W, p + "shared.", h, r)
    return out


# --------------------------------------------------------------------------- the model
def run_order(cfg):
    """(layer, number of the loop's pass that starts here or None) in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    order = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        order += [(i, t if i == a else None) for i in range(a, b)]
    return order + [(i, None) for i in range(b, n)]


def forward(cfg, W, ids, layers_out=None, r=exact, routes=None, slack=0.0):
    """Logits [T, V] of one whole sequence.  ``layers_out``: a list that receives the stream after every layer run.
    ``routes``: run -> position -> experts (see ``experts``)."""
    eps = cfg["norm"]["eps"]
    start = W["embed"][np.asarray(ids)] * cfg["embedding"]["scale"]
    x = start.copy()
    for run, (i, begins) in enumerate(run_order(cfg)):
        L, p = cfg["layers"][i], f"l{i}."
        if begins is not None:
            x = x + (start if begins else 0.0) + W["loop.step"][begins]
        h = r(layer_norm(x, W[p + "norm1"], eps))
        if L["type"] == "rglru":
            y = recurrent_block(W, p, h, r)
        elif L["type"] == "attention":
            y = attention(W, p, L["mixer"], h, r)
        else:
            raise ValueError(L["type"])
        if L.get("mlp"):
            y = y + experts(W, p + "mlp.", L["mlp"], h, r, None if routes is None else routes.get(run), slack)
        x = x + y
        if layers_out is not None:
            layers_out.append(x.copy())
    return r(layer_norm(x, W["final.norm"], eps)) @ W["embed"].T


def forward_logits(cfg, W, ids):
    return forward(cfg, W, ids)


def greedy_generate(cfg, W, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(np.argmax(forward(cfg, W, ids)[-1])))
    return ids[len(prompt):]
