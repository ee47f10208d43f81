"""Typed Mogevik configuration, read from the design's own config.json keys.

A Mogevik model is a list of layers.  Every layer has one layer norm (a gain, no bias) whose output both its mixer and its
feed-forward read; their results join the stream together.  The mixer is a gated linear recurrence with one real number of
state a channel (``rglru``), or softmax attention over a window with grouped key heads, biases on queries, keys and values,
scores that fall with the distance by a slope per head, and a logistic gate of the input on the heads' results
(``attention``).  The feed-forward, unless ``mlp`` is null, is a mixture of gated experts: a softmax over all router outputs
with a correction that only decides, optional groups, optional experts that hand their input on, and an optional shared
expert with a logistic gate a token.  A range of layers may run several times with the same weights; every pass keeps a
cache or state of its own and starts by adding the embedding output (from the second pass on) and a learned vector of the
pass to the stream.  The embedding is multiplied by a constant; the head is the embedding table.  config.json::

    {"architecture": "Mogevik", "vocab": V, "width": E, "norm": {"eps": e}, "embedding": {"scale": s},
     "loop": null | {"start": a, "stop": b, "times": n},
     "layers": [{"type": "rglru", "mixer": {"width", "blocks", "conv"},
                 "mlp": null | {"kind": "moe", "expert": {"ff"},
                                "router": {"experts", "top", "identity": n, "groups": null | {"count", "keep"}},
                                "shared": null | {"ff"}}},
                {"type": "attention",
                 "mixer": {"heads", "kv_heads", "dim", "vdim", "scale", "mask": null | {"size"}}, "mlp": ...}, ...]}
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional, Tuple

from .salivik import _float, _int, _Reader
from .specs import (AttentionSpec, ConfigError, ExpertsFeedForwardSpec, LayerCall, LayerSpec, ModelConfig, NormSpec,
                    PositionSpec, RealGatedRecurrenceSpec)

ARCHITECTURE = "Mogevik"
DEFAULT_MAX_POSITIONS = 1 << 20     # positions enter through distances only: requests are bounded by the cache
# fixed by the design
FF_ACTIVATION, BRANCH_ACTIVATION, DECAY_STRENGTH = "silu", "gelu_pytorch_tanh", 8.0
MIXERS = ("rglru", "attention")
_INTS = {"rglru": ("width", "blocks", "conv"), "attention": ("heads", "kv_heads", "dim", "vdim")}


def head_slopes(heads: int) -> Tuple[float, ...]:
    """What a score of head h loses for every position of distance: 2^(-8 (h + 1) / heads)."""
    return tuple(2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads))


@dataclass(frozen=True)
class MogevikFeedForward:
    ff: int
    experts: int
    top: int
    identity: int = 0
    groups: Optional[Tuple[int, int]] = None        # count, keep
    shared_ff: int = 0                              # 0: no shared expert

    @property
    def outputs(self) -> int:
        return self.experts + self.identity

    def to_dict(self) -> dict:
        router = {"experts": self.experts, "top": self.top}
        if self.identity:
            router["identity"] = self.identity
        if self.groups is not None:
            router["groups"] = {"count": self.groups[0], "keep": self.groups[1]}
        return {"kind": "moe", "expert": {"ff": self.ff}, "router": router,
                "shared": {"ff": self.shared_ff} if self.shared_ff else None}


@dataclass(frozen=True)
class MogevikLayer:
    kind: str                                 # "rglru" | "attention"
    sizes: Tuple[Tuple[str, int], ...]        # the mixer's integer sizes by their config names
    scale: float = 1.0                        # attention, as is the next
    window: Optional[int] = None
    mlp: Optional[MogevikFeedForward] = None

    def n(self, key: str) -> int:
        return dict(self.sizes)[key]

    def to_dict(self) -> dict:
        m = dict(self.sizes)
        if self.kind == "attention":
            m["scale"] = self.scale
            m["mask"] = None if self.window is None else {"size": self.window}
        return {"type": self.kind, "mixer": m, "mlp": None if self.mlp is None else self.mlp.to_dict()}


def _read_feed_forward(r: _Reader, mlp, w: str) -> Optional[MogevikFeedForward]:
    n0 = len(r.missing)
    kind = r.get(mlp, "kind", w)
    if kind is not None and kind != "moe":
        raise ConfigError(f"{w}kind is {kind!r}; this design's feed-forward: 'moe'")
    ex, ro = r.get(mlp, "expert", w), r.get(mlp, "router", w)
    ff = r.get(ex, "ff", w + "expert.") if ex is not None else None
    n = r.get(ro, "experts", w + "router.") if ro is not None else None
    top = r.get(ro, "top", w + "router.") if ro is not None else None
    gr = ro.get("groups") if isinstance(ro, dict) else None
    count = r.get(gr, "count", w + "router.groups.") if gr is not None else None
    keep = r.get(gr, "keep", w + "router.groups.") if gr is not None else None
    sh = mlp.get("shared") if isinstance(mlp, dict) else None
    sf = r.get(sh, "ff", w + "shared.") if sh is not None else None
    if len(r.missing) > n0:
        return None
    identity = ro.get("identity")
    return MogevikFeedForward(
        _int(ff, w + "expert.ff"), _int(n, w + "router.experts"), _int(top, w + "router.top"),
        identity=0 if identity is None else _int(identity, w + "router.identity", 0),
        groups=None if gr is None else (_int(count, w + "router.groups.count"), _int(keep, w + "router.groups.keep")),
        shared_ff=0 if sh is None else _int(sf, w + "shared.ff"))


def _read_layer(r: _Reader, L, w: str) -> Optional[MogevikLayer]:
    kind = r.get(L, "type", w)
    if kind is not None and kind not in MIXERS:
        raise ConfigError(f"{w}type is {kind!r}; this design's mixers: {', '.join(repr(k) for k in MIXERS)}")
    m = r.get(L, "mixer", w)
    if kind is None or m is None:
        return None
    n0, wm = len(r.missing), w + "mixer."
    ints = {k: r.get(m, k, wm) for k in _INTS[kind]}
    scale = size = None
    if kind == "attention":
        scale = r.get(m, "scale", wm)
        mask = m.get("mask") if isinstance(m, dict) else None
        size = r.get(mask, "size", wm + "mask.") if mask is not None else None
    mlp = L.get("mlp") if isinstance(L, dict) else None
    ff = _read_feed_forward(r, mlp, w + "mlp.") if mlp is not None else None
    if len(r.missing) > n0:
        return None
    return MogevikLayer(kind=kind, sizes=tuple((k, _int(v, wm + k)) for k, v in ints.items()),
                        scale=1.0 if scale is None else _float(scale, wm + "scale", positive=True),
                        window=None if size is None else _int(size, wm + "mask.size"), mlp=ff)


@dataclass(frozen=True)
class MogevikConfig:
    vocab: int
    width: int
    eps: float
    embed_scale: float
    layers: Tuple[MogevikLayer, ...]
    loop: Optional[Tuple[int, int, int]] = None       # start, stop, times
    max_positions: int = DEFAULT_MAX_POSITIONS
    bos_token_id: Optional[int] = None
    eos_token_id: Optional[int] = None

    @classmethod
    def from_dict(cls, d: dict) -> "MogevikConfig":
        r = _Reader()
        vocab, width = r.get(d, "vocab", ""), r.get(d, "width", "")
        norm, emb = r.get(d, "norm", ""), r.get(d, "embedding", "")
        eps = r.get(norm, "eps", "norm.") if norm is not None else None
        scale = r.get(emb, "scale", "embedding.") if emb is not None else None
        layers: List[MogevikLayer] = []
        for i, L in enumerate(r.get(d, "layers", "") or []):
            layer = _read_layer(r, L, f"layers[{i}].")
            if layer is not None:
                layers.append(layer)
        loop, lp = None, d.get("loop") if isinstance(d, dict) else None
        if lp is not None:
            vals = [r.get(lp, k, "loop.") for k in ("start", "stop", "times")]
            if all(v is not None for v in vals):
                loop = (_int(vals[0], "loop.start", 0), _int(vals[1], "loop.stop", 0), _int(vals[2], "loop.times"))
        if r.missing:
            raise ConfigError("Mogevik config.json lacks required keys: " + ", ".join(r.missing))
        cfg = cls(vocab=_int(vocab, "vocab"), width=_int(width, "width"), eps=_float(eps, "norm.eps", positive=True),
                  embed_scale=_float(scale, "embedding.scale"), layers=tuple(layers), loop=loop,
                  max_positions=_int(d.get("max_positions", DEFAULT_MAX_POSITIONS), "max_positions"),
                  bos_token_id=d.get("bos_token_id"), eos_token_id=d.get("eos_token_id"))
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if not self.layers:
            raise ConfigError("a Mogevik model needs at least one layer")
        if self.loop is not None:
            a, b, _ = self.loop
            if not (0 <= a < b <= len(self.layers)):
                raise ConfigError(f"loop.start {a} and loop.stop {b} must name a range of the {len(self.layers)} layers")
        for i, L in enumerate(self.layers):
            w = f"layers[{i}]"
            if L.kind == "rglru" and L.n("width") % L.n("blocks") != 0:
                raise ConfigError(f"{w}: {L.n('width')} channels do not fall into {L.n('blocks')} equal blocks")
            if L.kind == "attention" and L.n("heads") % L.n("kv_heads") != 0:
                raise ConfigError(f"{w}: {L.n('heads')} heads are not a multiple of {L.n('kv_heads')} key heads")
            f = L.mlp
            if f is None:
                continue
            can = f.outputs
            if f.groups is not None:
                count, keep = f.groups
                if f.outputs % count != 0 or keep > count:
                    raise ConfigError(f"{w}: {f.outputs} router outputs in {count} equal groups of which {keep} are kept")
                can = f.outputs // count * keep
            if f.top > can:
                raise ConfigError(f"{w}: top {f.top} of {can} experts that can be chosen")

    def to_dict(self) -> dict:
        d = {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
             "embedding": {"scale": self.embed_scale}, "layers": [L.to_dict() for L in self.layers],
             "loop": None if self.loop is None else dict(zip(("start", "stop", "times"), self.loop))}
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            d["max_positions"] = self.max_positions
        if self.bos_token_id is not None:
            d["bos_token_id"] = self.bos_token_id
        if self.eos_token_id is not None:
            d["eos_token_id"] = self.eos_token_id
        return d

    def run_order(self) -> List[Tuple[int, Optional[int]]]:
        """(layer, number of the loop's pass that starts here or None), in the order the layers run."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        a, b, times = self.loop
        order: List[Tuple[int, Optional[int]]] = [(i, None) for i in range(a)]
        for t in range(times):
            order += [(i, t if i == a else None) for i in range(a, b)]
        return order + [(i, None) for i in range(b, n)]

    # ---- the model as parts ------------------------------------------------------------------
    def to_model_config(self) -> ModelConfig:
        E = self.width
        norm = NormSpec("layernorm", E, self.eps, bias=False)
        specs = []
        for i, L in enumerate(self.layers):
            if L.kind == "rglru":
                mixer = RealGatedRecurrenceSpec("real_gated_recurrence", E, channels=L.n("width"), blocks=L.n("blocks"),
                                                conv_taps=L.n("conv"), decay_strength=DECAY_STRENGTH,
                                                activation=BRANCH_ACTIVATION)
            else:
                mixer = AttentionSpec(
                    "attention", E, L.n("heads"), L.n("kv_heads"), L.n("dim"), scale=L.scale, qkv_bias=True, out_bias=False,
                    window=L.window, v_head_dim=L.n("vdim"), out_gate="sigmoid", distance_slopes=head_slopes(L.n("heads")))
            f, ff = L.mlp, None
            if f is not None:
                count, keep = f.groups if f.groups is not None else (0, 0)
                ff = ExpertsFeedForwardSpec("experts", E, f.ff, f.experts, f.top, FF_ACTIVATION, router="softmax_all",
                                            groups=count, groups_kept=keep, identity=f.identity, shared_inner=f.shared_ff,
                                            shared_activation=FF_ACTIVATION, shared_gated=True, shared_token_gate=True)
            specs.append(LayerSpec(mixer=mixer, feed_forward=ff, pre_mixer_norm=norm, weight_prefix=f"l{i}.",
                                   parallel=ff is not None))
        # every run of a layer has a cache slot or state of its own
        schedule = tuple(LayerCall(layer, run, add_input=begins is not None and begins > 0, add_step=begins)
                         for run, (layer, begins) in enumerate(self.run_order()))
        eos = () if self.eos_token_id is None else (int(self.eos_token_id),)
        return ModelConfig(
            architecture=ARCHITECTURE, vocab_size=self.vocab, width=E, max_positions=self.max_positions,
            layers=tuple(specs), schedule=schedule, embed_position=PositionSpec("none"), final_norm=norm,
            tie_word_embeddings=True, bos_token_id=self.bos_token_id, eos_token_ids=eos, raw=self.to_dict(),
            embed_scale=self.embed_scale, step_vectors=0 if self.loop is None else self.loop[2])
