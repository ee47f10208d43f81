"""Typed Luvatar configuration, read from the design's own config.json keys.

A Luvatar model is a list of layers.  Every layer has a mixer that reads the residual stream itself (no norm in front)
and a root-mean-square norm behind it; then, unless its ``mlp`` is null, a gated feed-forward wired the same way.  The
mixer is gated linear attention with a decay per key channel (``gla``), or softmax attention inside chunks of positions
(``attention``) with grouped key heads, a norm of queries and keys head by head, rotations whose speeds may all be
divided by a factor, a learned term per head in the denominator and a logistic gate of the input on the heads' results.
An attention layer may name an earlier one in ``kv_from``: it then reads that layer's keys and values, with queries and
chunks of its own.  The embedding is multiplied by a constant; the head is the embedding table.  config.json::

    {"architecture": "Luvatar", "vocab": V, "width": E, "norm": {"eps": e}, "embedding": {"scale": s},
     "layers": [{"type": "gla", "mixer": {"heads", "dim", "vdim", "tau"},
                 "mlp": null | {"kind": "dense", "ff": F}},
                {"type": "attention",
                 "mixer": {"heads", "kv_heads", "dim", "vdim", "scale", "mask": null | {"size"},
                           "rot": null | {"base", "dims", "scaling": null | {"factor"}}, "kv_from": null | layer},
                 "mlp": ...}, ...]}

The low rank of a ``gla`` mixer's decay is the checkpoint's to say (its tensors' shapes); a config.json may name it as
``mixer.a_rank``, which the random-weights mode needs.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional, Tuple

from .salivik import _float, _int, _Reader
from .specs import (AttentionSpec, ConfigError, GatedFeedForwardSpec, GatedLinearSpec, LayerCall, LayerSpec,
                    LinearSpeedsSpec, ModelConfig, NormSpec, PositionSpec, QKNormSpec, RotarySpec)

ARCHITECTURE = "Luvatar"
DEFAULT_MAX_POSITIONS = 1 << 20     # positions enter through angles only: requests are bounded by the cache
FF_ACTIVATION = "silu"              # fixed by the design
MIXERS = ("gla", "attention")

_GLA_INTS = ("heads", "dim", "vdim")
_ATT_INTS = ("heads", "kv_heads", "dim", "vdim")


@dataclass(frozen=True)
class LuvatarRotation:
    base: float
    dims: int
    factor: Optional[float] = None      # scaling.factor: every speed is divided by it

    def to_dict(self) -> dict:
        d = {"base": self.base, "dims": self.dims}
        if self.factor is not None:
            d["scaling"] = {"factor": self.factor}
        return d

    def spec(self) -> RotarySpec:
        return RotarySpec("rotary", dims=self.dims, base=self.base, interleaved=True,
                          scaling=None if self.factor is None else LinearSpeedsSpec(self.factor))


@dataclass(frozen=True)
class LuvatarLayer:
    kind: str                                 # "gla" | "attention"
    sizes: Tuple[Tuple[str, int], ...]        # the mixer's integer sizes by their config names
    tau: float = 1.0                          # gla
    a_rank: int = -1                          # gla; -1: as the checkpoint's tensors say
    scale: float = 1.0                        # attention, as are the rest
    chunk: Optional[int] = None
    rot: Optional[LuvatarRotation] = None
    kv_from: Optional[int] = None
    ff: int = 0                               # 0: no feed-forward

    def n(self, key: str) -> int:
        return dict(self.sizes)[key]

    def to_dict(self) -> dict:
        m = dict(self.sizes)
        if self.kind == "gla":
            m["tau"] = self.tau
            if self.a_rank > 0:
                m["a_rank"] = self.a_rank
        else:
            m["scale"] = self.scale
            m["mask"] = None if self.chunk is None else {"size": self.chunk}
            m["rot"] = None if self.rot is None else self.rot.to_dict()
            if self.kv_from is not None:
                m["kv_from"] = self.kv_from
        return {"type": self.kind, "mixer": m, "mlp": {"kind": "dense", "ff": self.ff} if self.ff else None}


def _read_rotation(r: _Reader, rot, w: str) -> Optional[LuvatarRotation]:
    n0 = len(r.missing)
    base, dims = r.get(rot, "base", w), r.get(rot, "dims", w)
    sc = rot.get("scaling") if isinstance(rot, dict) else None
    factor = r.get(sc, "factor", w + "scaling.") if sc is not None else None
    if len(r.missing) > n0:
        return None
    return LuvatarRotation(_float(base, w + "base", positive=True), _int(dims, w + "dims", 0),
                           None if factor is None else _float(factor, w + "scaling.factor", positive=True))


def _read_layer(r: _Reader, L, w: str) -> Optional[LuvatarLayer]:
    kind = r.get(L, "type", w)
    if kind is not None and kind not in MIXERS:
        raise ConfigError(f"{w}type is {kind!r}; this design's mixers: {', '.join(repr(k) for k in MIXERS)}")
    m = r.get(L, "mixer", w)
    if kind is None or m is None:
        return None
    n0, wm = len(r.missing), w + "mixer."
    ints = {k: r.get(m, k, wm) for k in (_GLA_INTS if kind == "gla" else _ATT_INTS)}
    own = {}
    if kind == "gla":
        tau = r.get(m, "tau", wm)
    else:
        scale = r.get(m, "scale", wm)
        mask, rot = (m.get("mask"), m.get("rot")) if isinstance(m, dict) else (None, None)
        size = r.get(mask, "size", wm + "mask.") if mask is not None else None
        turn = _read_rotation(r, rot, wm + "rot.") if rot is not None else None
    mlp = L.get("mlp") if isinstance(L, dict) else None
    ff = 0
    if mlp is not None:
        ff_kind, ff = r.get(mlp, "kind", w + "mlp."), r.get(mlp, "ff", w + "mlp.")
        if ff_kind is not None and ff_kind != "dense":
            raise ConfigError(f"{w}mlp.kind is {ff_kind!r}; this design's feed-forward: 'dense'")
    if len(r.missing) > n0:
        return None
    if kind == "gla":
        own["tau"] = _float(tau, wm + "tau", positive=True)
        if m.get("a_rank") is not None:
            own["a_rank"] = _int(m["a_rank"], wm + "a_rank")
    else:
        own.update(scale=_float(scale, wm + "scale", positive=True), rot=turn,
                   chunk=None if size is None else _int(size, wm + "mask.size"),
                   kv_from=None if m.get("kv_from") is None else _int(m["kv_from"], wm + "kv_from", 0))
    return LuvatarLayer(kind=kind, sizes=tuple((k, _int(v, wm + k)) for k, v in ints.items()),
                        ff=_int(ff, w + "mlp.ff") if mlp is not None else 0, **own)


@dataclass(frozen=True)
class LuvatarConfig:
    vocab: int
    width: int
    eps: float
    embed_scale: float
    layers: Tuple[LuvatarLayer, ...]
    max_positions: int = DEFAULT_MAX_POSITIONS
    bos_token_id: Optional[int] = None
    eos_token_id: Optional[int] = None

    @classmethod
    def from_dict(cls, d: dict) -> "LuvatarConfig":
        r = _Reader()
        vocab, width = r.get(d, "vocab", ""), r.get(d, "width", "")
        norm, emb = r.get(d, "norm", ""), r.get(d, "embedding", "")
        eps = r.get(norm, "eps", "norm.") if norm is not None else None
        scale = r.get(emb, "scale", "embedding.") if emb is not None else None
        raw = r.get(d, "layers", "")
        layers: List[LuvatarLayer] = []
        for i, L in enumerate(raw or []):
            layer = _read_layer(r, L, f"layers[{i}].")
            if layer is not None:
                layers.append(layer)
        if r.missing:
            raise ConfigError("Luvatar config.json lacks required keys: " + ", ".join(r.missing))
        cfg = cls(vocab=_int(vocab, "vocab"), width=_int(width, "width"), eps=_float(eps, "norm.eps", positive=True),
                  embed_scale=_float(scale, "embedding.scale"), layers=tuple(layers),
                  max_positions=_int(d.get("max_positions", DEFAULT_MAX_POSITIONS), "max_positions"),
                  bos_token_id=d.get("bos_token_id"), eos_token_id=d.get("eos_token_id"))
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if not self.layers:
            raise ConfigError("a Luvatar model needs at least one layer")
        for i, L in enumerate(self.layers):
            w = f"layers[{i}]"
            if L.kind != "attention":
                continue
            if L.n("heads") % L.n("kv_heads") != 0:
                raise ConfigError(f"{w}: {L.n('heads')} heads are not a multiple of {L.n('kv_heads')} key heads")
            if L.rot is not None and (L.rot.dims % 2 != 0 or L.rot.dims > L.n("dim")):
                raise ConfigError(f"{w}: rot.dims {L.rot.dims} must be even and at most {L.n('dim')}")
            if L.kv_from is None:
                continue
            if not L.kv_from < i or self.layers[L.kv_from].kind != "attention":
                raise ConfigError(f"{w}: kv_from {L.kv_from} must name an earlier attention layer")
            other = self.layers[L.kv_from]
            if other.kv_from is not None:
                raise ConfigError(f"{w}: kv_from {L.kv_from} names a layer that has no keys and values of its own")
            if any(L.n(k) != other.n(k) for k in ("kv_heads", "dim", "vdim")) or L.rot != other.rot:
                raise ConfigError(f"{w}: key heads, head sizes and rotation differ from layer {L.kv_from}'s, whose keys it reads")

    def to_dict(self) -> dict:
        d = {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
             "embedding": {"scale": self.embed_scale}, "layers": [L.to_dict() for L in self.layers]}
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            d["max_positions"] = self.max_positions
        if self.bos_token_id is not None:
            d["bos_token_id"] = self.bos_token_id
        if self.eos_token_id is not None:
            d["eos_token_id"] = self.eos_token_id
        return d

    # ---- the model as parts ------------------------------------------------------------------
    def to_model_config(self) -> ModelConfig:
        E = self.width
        norm = NormSpec("rmsnorm", E, self.eps, bias=False, gain_offset=0.0)
        specs, schedule = [], []
        for i, L in enumerate(self.layers):
            if L.kind == "gla":
                mixer = GatedLinearSpec("gated_linear", E, L.n("heads"), L.n("dim"), L.n("vdim"), tau=L.tau,
                                        norm_eps=self.eps, decay_rank=L.a_rank, gate="silu")
            else:
                mixer = AttentionSpec(
                    "attention", E, L.n("heads"), L.n("kv_heads"), L.n("dim"), scale=L.scale, qkv_bias=False, out_bias=False,
                    position=None if L.rot is None else L.rot.spec(), v_head_dim=L.n("vdim"), chunk=L.chunk,
                    qk_norm=QKNormSpec(self.eps, whole=False), sink="learned", out_gate="sigmoid",
                    shared_kv=L.kv_from is not None)
            ff = GatedFeedForwardSpec("gated", E, L.ff, FF_ACTIVATION) if L.ff else None
            specs.append(LayerSpec(mixer=mixer, feed_forward=ff, post_mixer_norm=norm,
                                   post_ff_norm=None if ff is None else norm, weight_prefix=f"l{i}."))
            # a layer has the cache slot of its number; one on another layer's keys and values reads that layer's slot
            schedule.append(LayerCall(i, i) if L.kv_from is None else LayerCall(i, L.kv_from, write=False))
        eos = () if self.eos_token_id is None else (int(self.eos_token_id),)
        return ModelConfig(
            architecture=ARCHITECTURE, vocab_size=self.vocab, width=E, max_positions=self.max_positions,
            layers=tuple(specs), schedule=tuple(schedule), embed_position=PositionSpec("none"), final_norm=norm,
            tie_word_embeddings=True, bos_token_id=self.bos_token_id, eos_token_ids=eos, raw=self.to_dict(),
            embed_scale=self.embed_scale)
