"""Luvatar: which checkpoint tensors feed which part.

Names: ``embed``, ``final.norm``; per layer ``l<i>.norm1`` and, with a feed-forward, ``l<i>.norm2``, ``l<i>.mlp.{gate,
up, down}``.  A gated linear mixer ``l<i>.mix.{q, k, v, g, o, norm, a1, a2}`` and ``l<i>.mix.a2.b``; an attention mixer
``l<i>.mix.{q, k, v, g, o, sink}`` and the gains ``l<i>.mix.{q, k}.norm``; one on another layer's keys and values has no
k, v and k.norm.  Linear weights are stored [out, in].  q | k | v | gate of an attention mixer (q | gate without keys
of its own) and gate | up of a feed-forward become one matrix each at load time.  The head is the embedding table.
"""
from __future__ import annotations

from typing import List

import torch

from ..config.luvatar import ARCHITECTURE, LuvatarConfig
from ..config.specs import AttentionSpec, GatedLinearSpec, ModelConfig
from ..registry import Architecture, ModelSupport
from ..weights.loader import TensorDecl

# Random-weights distributions: matrices N(0, 0.05) (queries and keys twice, the decay's second factor four times that),
# norm gains 1 + N(0, 0.1), the decay's bias and the sinks N(0, 1) and N(0, 0.5).
W_STD, GAIN_STD = 0.05, 0.1


def read_config(d: dict) -> ModelConfig:
    return LuvatarConfig.from_dict(d).to_model_config()


def _gated_linear_decls(p: str, m: GatedLinearSpec, E: int) -> List[TensorDecl]:
    qk, v, r = m.n_heads * m.head_dim, m.n_heads * m.v_head_dim, m.decay_rank
    return [TensorDecl(p + "q", (qk, E), "normal", 2 * W_STD), TensorDecl(p + "k", (qk, E), "normal", 2 * W_STD),
            TensorDecl(p + "v", (v, E), "normal", W_STD), TensorDecl(p + "g", (v, E), "normal", W_STD),
            TensorDecl(p + "o", (E, v), "normal", W_STD), TensorDecl(p + "norm", (m.v_head_dim,), "ones_plus_normal", GAIN_STD),
            TensorDecl(p + "a1", (r, E), "normal", W_STD), TensorDecl(p + "a2", (qk, r), "normal", 4 * W_STD),
            TensorDecl(p + "a2.b", (qk,), "normal", 1.0)]


def _attention_decls(p: str, m: AttentionSpec, E: int) -> List[TensorDecl]:
    H, G, D, Dv = m.n_heads, m.n_kv_heads, m.head_dim, m.value_dim
    out = [TensorDecl(p + "q", (H * D, E), "normal", 2 * W_STD), TensorDecl(p + "q.norm", (D,), "ones_plus_normal", GAIN_STD),
           TensorDecl(p + "sink", (H,), "normal", 0.5), TensorDecl(p + "g", (H * Dv, E), "normal", W_STD),
           TensorDecl(p + "o", (E, H * Dv), "normal", W_STD)]
    if not m.shared_kv:
        out += [TensorDecl(p + "k", (G * D, E), "normal", 2 * W_STD), TensorDecl(p + "v", (G * Dv, E), "normal", W_STD),
                TensorDecl(p + "k.norm", (D,), "ones_plus_normal", GAIN_STD)]
    return out


def declare_tensors(mc: ModelConfig) -> List[TensorDecl]:
    E, V = mc.width, mc.vocab_size
    out = [TensorDecl("embed", (V, E), "normal", 0.3)]
    for spec in mc.layers:
        p, m, f = spec.weight_prefix, spec.mixer, spec.feed_forward
        out.append(TensorDecl(p + "norm1", (E,), "ones_plus_normal", GAIN_STD))
        if isinstance(m, GatedLinearSpec):
            out += _gated_linear_decls(p + "mix.", m, E)
        elif isinstance(m, AttentionSpec):
            out += _attention_decls(p + "mix.", m, E)
        else:
            raise TypeError(f"no tensors are known for a mixer of kind {getattr(m, 'kind', m)!r}")
        if f is not None:
            out += [TensorDecl(p + "norm2", (E,), "ones_plus_normal", GAIN_STD),
                    TensorDecl(p + "mlp.gate", (f.inner, E), "normal", W_STD),
                    TensorDecl(p + "mlp.up", (f.inner, E), "normal", W_STD),
                    TensorDecl(p + "mlp.down", (E, f.inner), "normal", W_STD)]
    out.append(TensorDecl("final.norm", (E,), "ones_plus_normal", GAIN_STD))
    return out


def bind_tensors(mc: ModelConfig, t: dict) -> dict:
    layers = []
    for spec in mc.layers:
        p, m, f = spec.weight_prefix, spec.mixer, spec.feed_forward
        d = {"post_mixer_norm": {"weight": t[p + "norm1"]}}
        w = lambda name: t[p + "mix." + name]
        if isinstance(m, GatedLinearSpec):
            d["mixer"] = {"q_weight": w("q"), "k_weight": w("k"), "v_weight": w("v"), "gate_weight": w("g"),
                          "decay_down": w("a1"), "decay_up": w("a2"), "decay_bias": w("a2.b"), "out_norm": w("norm"),
                          "out_weight": w("o")}
        else:
            rows = ("q", "g") if m.shared_kv else ("q", "k", "v", "g")
            d["mixer"] = {"qkv_weight": torch.cat([w(n) for n in rows], 0), "out_weight": w("o"), "sink": w("sink"),
                          "q_norm": w("q.norm")}
            if not m.shared_kv:
                d["mixer"]["k_norm"] = w("k.norm")
        if f is not None:
            d["post_ff_norm"] = {"weight": t[p + "norm2"]}
            d["feed_forward"] = {"gate_up_weight": torch.cat([t[p + "mlp.gate"], t[p + "mlp.up"]], 0),
                                 "down_weight": t[p + "mlp.down"]}
        layers.append(d)
    return {"embed": {"tokens": t["embed"]}, "layers": layers, "final_norm": {"weight": t["final.norm"]},
            "head": {"weight": t["embed"]}}


LUVATAR = Architecture(name=ARCHITECTURE, read_config=read_config, declare_tensors=declare_tensors,
                       bind_tensors=bind_tensors, aliases=("luvatar",))
ModelSupport.add_model(LUVATAR)
