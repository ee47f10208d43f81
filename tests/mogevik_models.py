"""Small Mogevik configurations for the tests, each different in every size and option, and a model folder with
random weights beside its plain implementation."""
from __future__ import annotations

import functools

import numpy as np

import plain_mogevik as P


def rec(width, blocks, conv):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}}


def att(heads, kv_heads, dim, vdim, scale, window):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                                           "mask": None if window is None else {"size": window}}}


def moe(experts, top, ff, identity=0, groups=None, shared=None):
    router = {"experts": experts, "top": top}
    if identity:
        router["identity"] = identity
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": router, "shared": None if shared is None else {"ff": shared}}


def layer(mixer, mlp=None):
    return dict(mixer, mlp=mlp)


def config(vocab, width, eps, scale, layers, loop=None):
    return {"architecture": "Mogevik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": layers, "loop": None if loop is None else dict(zip(("start", "stop", "times"), loop))}


# D: both mixers with and without a feed-forward; blocks of 16 and of 96 channels; groups with experts that hand their
# input on among them; a shared expert whose size is a multiple of the others' and one whose size is not; values larger
# than keys; windows that are no multiple of a page; a loop of three passes in the middle
CONFIG_D = config(300, 64, 1e-5, 3.0,
                  [layer(rec(48, 3, 4), moe(7, 3, 24, identity=2, groups=(3, 2), shared=48)),
                   layer(att(4, 2, 16, 24, 0.3, 20), moe(4, 2, 32, shared=40)),
                   layer(rec(96, 1, 2)),
                   layer(att(6, 6, 32, 32, 0.15, 45), moe(5, 1, 16, identity=1, groups=(2, 1)))],
                  loop=(1, 3, 3))

# E: sizes that are no multiple of 8 (plain products, plain attention and the walking form of the recurrence); one key
# head for all query heads; as many experts a token as there are; every group kept; no loop
CONFIG_E = config(130, 52, 1e-6, 0.7,
                  [layer(rec(60, 5, 3), moe(3, 4, 20, identity=1, groups=(2, 2), shared=12)),
                   layer(att(3, 1, 12, 20, 0.4, 64)),
                   layer(rec(36, 2, 6), moe(3, 2, 28))])

# F: the ones: one block, one tap, one head, one expert, embedding scale 1, a window of one key (a token sees itself
# only) and none at all; more experts that hand their input on than others; a loop over all layers that starts at the
# first one
CONFIG_F = config(64, 48, 1e-5, 1.0,
                  [layer(rec(40, 1, 1), moe(1, 1, 40)),
                   layer(att(1, 1, 40, 16, 0.2, 1), moe(2, 2, 16, identity=4, groups=(1, 1), shared=16)),
                   layer(att(2, 2, 24, 24, 0.25, None), moe(2, 1, 24, identity=6, groups=(4, 1)))],
                  loop=(0, 3, 2))


class TinyMogevik:
    def __init__(self, folder, cfg, seed):
        self.folder, self.cfg, self.seed = str(folder), cfg, seed
        self.plain_cfg, self.W = P.read_model_folder(self.folder)

    @functools.lru_cache(maxsize=None)
    def _logits(self, ids):
        return P.forward_logits(self.plain_cfg, self.W, list(ids))

    def plain_logits(self, ids, routes=None, slack=0.0):
        """The plain model's logits [T, V]; with ``routes`` (run -> position -> experts chosen by the engine) it makes
        the engine's choices where they are as good as its own within ``slack``."""
        if routes is None:
            return self._logits(tuple(int(i) for i in ids))
        return P.forward(self.plain_cfg, self.W, list(ids), routes=routes, slack=slack)

    def prompt(self, length, salt=0):
        rng = np.random.default_rng(1000 * self.seed + 7 * length + salt)
        return [int(t) for t in rng.integers(0, self.cfg["vocab"], size=length)]


def make_model(folder, cfg, seed):
    from deliverance_amd.random_model import random_model
    random_model(str(folder), cfg, seed)
    return TinyMogevik(folder, cfg, seed)


def replay_routed(session, steps, cfg):
    """helpers.replay, and beside the logits the experts that the engine chose: {rid: {run: {position: [experts]}}}.
    The engine hands them to its layer debug hook once per run of a layer with a feed-forward, rows in the step's order
    (one-token entries first, then the portions, each group in the order of the entries)."""
    got, routes, at, seen = {}, {}, {}, []
    session.runner.debug_hook = lambda layer_, stage, t: seen.append(t.cpu().numpy()) if stage == "expert_choice" else None
    runs = [run for run, (i, _) in enumerate(P.run_order(cfg)) if cfg["layers"][i].get("mlp")]
    try:
        for s in steps:
            seen.clear()
            out, r = session.run_step(s), 0
            for e in s["entries"]:
                for _ in e.get("want", []):
                    got.setdefault(e["id"], []).append(out[r])
                    r += 1
            assert len(seen) == len(runs), f"{len(seen)} feed-forwards reported, the model runs {len(runs)}"
            row = 0
            for e in sorted(s["entries"], key=lambda e: len(e["tokens"]) != 1):
                start, n = at.get(e["id"], 0), len(e["tokens"])
                for run, ids in zip(runs, seen):
                    of = routes.setdefault(e["id"], {}).setdefault(run, {})
                    of.update({start + j: [int(x) for x in ids[row + j]] for j in range(n)})
                row += n
                at[e["id"]] = start + n
            for rid in s["end"]:
                at.pop(rid, None)
    finally:
        session.runner.debug_hook = None
    return {rid: np.stack(rows) for rid, rows in got.items()}, routes
