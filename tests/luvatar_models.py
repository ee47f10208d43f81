"""Small Luvatar configurations for the tests, each different in every size and option, and a model folder with
random weights beside its plain implementation."""
from __future__ import annotations

import functools

import numpy as np

import plain_luvatar as P


def rot(base, dims, factor=None):
    d = {"base": base, "dims": dims}
    if factor is not None:
        d["scaling"] = {"factor": factor}
    return d


def gla(heads, dim, vdim, tau, a_rank):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "a_rank": a_rank}}


def att(heads, kv_heads, dim, vdim, scale, chunk, turn, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
         "mask": None if chunk is None else {"size": chunk}, "rot": turn}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m}


def layer(mixer, ff=None):
    return dict(mixer, mlp=None if ff is None else {"kind": "dense", "ff": ff})


def config(vocab, width, eps, scale, layers):
    return {"architecture": "Luvatar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": layers}


# A: both mixers with and without a feed-forward; values smaller than keys; a layer on another's keys with longer chunks
# than that layer's; part of a head turns, at a third of the speed; chunks that are no multiple of a page
CONFIG_A = config(300, 64, 1e-5, 3.0,
                  [layer(att(4, 2, 16, 8, 0.3, 20, rot(10000.0, 8, 3.0)), 96),
                   layer(gla(3, 16, 24, 4.0, 8)),
                   layer(att(4, 2, 16, 8, 0.2, 50, rot(10000.0, 8, 3.0), kv_from=0)),
                   layer(gla(2, 32, 16, 16.0, 12), 40)])

# B: sizes that are no multiple of 8 (plain products, plain attention and the walking form of the recurrence); one key
# head for all query heads; values larger than keys; no scaling; the reading layer has shorter chunks and other query
# heads than its source, and is read twice; a fast decay (tau below 1) through a rank that is no multiple of 4
CONFIG_B = config(130, 52, 1e-6, 0.7,
                  [layer(gla(2, 18, 10, 0.5, 5), 36),
                   layer(att(3, 1, 12, 20, 0.4, 64, rot(500.0, 12)), 28),
                   layer(att(2, 1, 12, 20, 0.5, 7, rot(500.0, 12), kv_from=1), 20),
                   layer(att(3, 1, 12, 20, 0.3, None, rot(500.0, 12), kv_from=1))])

# C: the ones: one head everywhere, tau 1, embedding scale 1, as many key heads as query heads, a factor of 1, chunks of
# one position (a token sees itself only) and of more than any prompt; nothing turns in one layer
CONFIG_C = config(64, 48, 1e-5, 1.0,
                  [layer(gla(1, 20, 36, 1.0, 4), 24),
                   layer(att(2, 2, 24, 24, 0.25, 1, rot(100.0, 24, 1.0)), 32),
                   layer(att(1, 1, 40, 16, 0.2, 1000, rot(100.0, 0)), 16),
                   layer(gla(4, 8, 8, 2.5, 40))])


class TinyLuvatar:
    def __init__(self, folder, cfg, seed):
        self.folder, self.cfg, self.seed = str(folder), cfg, seed
        self.plain_cfg, self.W = P.read_model_folder(self.folder)

    @functools.lru_cache(maxsize=None)
    def _logits(self, ids):
        return P.forward_logits(self.plain_cfg, self.W, list(ids))

    def plain_logits(self, ids):
        return self._logits(tuple(int(i) for i in ids))

    @functools.lru_cache(maxsize=None)
    def _rounded(self, ids):
        import torch
        return P.forward(self.plain_cfg, self.W, list(ids), r=lambda x: torch.tensor(x).to(torch.bfloat16).double().numpy())

    def rounding_error(self, ids):
        """[T]: how far rounding to bfloat16 alone moves a position's logits (root mean square over the vocabulary)."""
        ids = tuple(int(i) for i in ids)
        return np.sqrt(((self._rounded(ids) - self._logits(ids)) ** 2).mean(axis=1))

    def prompt(self, length, salt=0):
        rng = np.random.default_rng(1000 * self.seed + 7 * length + salt)
        return [int(t) for t in rng.integers(0, self.cfg["vocab"], size=length)]


def make_model(folder, cfg, seed):
    from deliverance_amd.random_model import random_model
    random_model(str(folder), cfg, seed)
    return TinyLuvatar(folder, cfg, seed)
