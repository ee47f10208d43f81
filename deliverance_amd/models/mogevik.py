"""Mogevik: which checkpoint tensors feed which part.

Names: ``embed``, ``final.norm``, with a loop ``loop.step``; per layer ``l<i>.norm1``.  A recurrent mixer
``l<i>.mix.{y, x, conv, ra, ri}`` with their biases ``.b``, ``l<i>.mix.lam`` and ``l<i>.mix.o``; an attention mixer
``l<i>.mix.{q, k, v}`` with their biases, ``l<i>.mix.{g, o}``; a feed-forward ``l<i>.mlp.router``, ``l<i>.mlp.correction``,
``l<i>.mlp.e<j>.{gate, up, down}`` and, with a shared expert, ``l<i>.mlp.shared.{gate, up, down, sg}``.  Linear weights are
stored [out, in].  y | x of a recurrent mixer, its two square matrices block by block, q | k | v | gate of an attention
mixer, gate | up of an expert, the experts of a layer, and router | shared gate become one matrix or stack each at load
time.  The head is the embedding table.
"""
from __future__ import annotations

from typing import List

import torch

from ..config.mogevik import ARCHITECTURE, MogevikConfig
from ..config.specs import AttentionSpec, ExpertsFeedForwardSpec, ModelConfig, RealGatedRecurrenceSpec
from ..registry import Architecture, ModelSupport
from ..weights.loader import TensorDecl

# Random-weights distributions: matrices N(0, 0.1) (routers and the shared expert's gate twice that), norm gains
# 1 + N(0, 0.1), biases N(0, 0.1), the recurrence's rates and square matrices N(0, 1) and N(0, 0.2).
W_STD, GAIN_STD = 0.1, 0.1


def read_config(d: dict) -> ModelConfig:
    return MogevikConfig.from_dict(d).to_model_config()


def _gated(p: str, inner: int, E: int) -> List[TensorDecl]:
    return [TensorDecl(p + "gate", (inner, E), "normal", W_STD), TensorDecl(p + "up", (inner, E), "normal", W_STD),
            TensorDecl(p + "down", (E, inner), "normal", W_STD)]


def _recurrence_decls(p: str, m: RealGatedRecurrenceSpec, E: int) -> List[TensorDecl]:
    C, B, n = m.channels, m.blocks, m.channels // m.blocks
    return [TensorDecl(p + "y", (C, E), "normal", W_STD), TensorDecl(p + "y.b", (C,), "normal", GAIN_STD),
            TensorDecl(p + "x", (C, E), "normal", W_STD), TensorDecl(p + "x.b", (C,), "normal", GAIN_STD),
            TensorDecl(p + "conv", (C, m.conv_taps), "normal", 0.5), TensorDecl(p + "conv.b", (C,), "normal", GAIN_STD),
            TensorDecl(p + "ra", (B, n, n), "normal", 0.2), TensorDecl(p + "ra.b", (B, n), "normal", 0.5),
            TensorDecl(p + "ri", (B, n, n), "normal", 0.2), TensorDecl(p + "ri.b", (B, n), "normal", 0.5),
            TensorDecl(p + "lam", (C,), "normal", 1.0), TensorDecl(p + "o", (E, C), "normal", W_STD)]


def _attention_decls(p: str, m: AttentionSpec, E: int) -> List[TensorDecl]:
    H, G, D, Dv = m.n_heads, m.n_kv_heads, m.head_dim, m.value_dim
    out = []
    for name, rows in (("q", H * D), ("k", G * D), ("v", G * Dv)):
        out += [TensorDecl(p + name, (rows, E), "normal", W_STD), TensorDecl(p + name + ".b", (rows,), "normal", GAIN_STD)]
    return out + [TensorDecl(p + "g", (H * Dv, E), "normal", W_STD), TensorDecl(p + "o", (E, H * Dv), "normal", W_STD)]


def _experts_decls(p: str, f: ExpertsFeedForwardSpec, E: int) -> List[TensorDecl]:
    out: List[TensorDecl] = []
    for j in range(f.n_experts):
        out += _gated(f"{p}e{j}.", f.inner, E)
    n = f.n_experts + f.identity
    out += [TensorDecl(p + "router", (n, E), "normal", 2 * W_STD), TensorDecl(p + "correction", (n,), "normal", 0.1)]
    if f.shared_inner:
        out += _gated(p + "shared.", f.shared_inner, E) + [TensorDecl(p + "shared.sg", (1, E), "normal", 2 * W_STD)]
    return out


def declare_tensors(mc: ModelConfig) -> List[TensorDecl]:
    E, V = mc.width, mc.vocab_size
    out = [TensorDecl("embed", (V, E), "normal", 0.3)]
    if mc.step_vectors:
        out.append(TensorDecl("loop.step", (mc.step_vectors, E), "normal", 0.3))
    for spec in mc.layers:
        p, m, f = spec.weight_prefix, spec.mixer, spec.feed_forward
        out.append(TensorDecl(p + "norm1", (E,), "ones_plus_normal", GAIN_STD))
        if isinstance(m, RealGatedRecurrenceSpec):
            out += _recurrence_decls(p + "mix.", m, E)
        elif isinstance(m, AttentionSpec):
            out += _attention_decls(p + "mix.", m, E)
        else:
            raise TypeError(f"no tensors are known for a mixer of kind {getattr(m, 'kind', m)!r}")
        if f is not None:
            out += _experts_decls(p + "mlp.", f, E)
    out.append(TensorDecl("final.norm", (E,), "ones_plus_normal", GAIN_STD))
    return out


def bind_tensors(mc: ModelConfig, t: dict) -> dict:
    layers = []
    for spec in mc.layers:
        p, m, f = spec.weight_prefix, spec.mixer, spec.feed_forward
        d = {"pre_mixer_norm": {"weight": t[p + "norm1"]}}
        w = lambda name: t[p + "mix." + name]
        if isinstance(m, RealGatedRecurrenceSpec):
            d["mixer"] = {"in_weight": torch.cat([w("y"), w("x")], 0), "in_bias": torch.cat([w("y.b"), w("x.b")], 0),
                          "conv_weight": w("conv"), "conv_bias": w("conv.b"),
                          "gate_weight": torch.cat([w("ra"), w("ri")], 1), "gate_bias": torch.cat([w("ra.b"), w("ri.b")], 1),
                          "lam": w("lam"), "out_weight": w("o")}
        else:
            # the gate's rows ride behind q | k | v; they have no bias
            gate = w("g")
            d["mixer"] = {"qkv_weight": torch.cat([w("q"), w("k"), w("v"), gate], 0), "out_weight": w("o"),
                          "qkv_bias": torch.cat([w("q.b"), w("k.b"), w("v.b"), w("q.b").new_zeros(gate.shape[0])])}
        if f is not None:
            q = p + "mlp."
            both = lambda e: torch.cat([t[e + "gate"], t[e + "up"]], 0)
            ff = {"gate_up_weight": torch.stack([both(f"{q}e{j}.") for j in range(f.n_experts)]),
                  "down_weight": torch.stack([t[f"{q}e{j}.down"] for j in range(f.n_experts)]),
                  "router_weight": t[q + "router"], "router_correction": t[q + "correction"]}
            if f.shared_inner:
                ff.update(shared_gate_up_weight=both(q + "shared."), shared_down_weight=t[q + "shared.down"],
                          shared_token_gate=t[q + "shared.sg"])
            d["feed_forward"] = ff
        layers.append(d)
    out = {"embed": {"tokens": t["embed"]}, "layers": layers, "final_norm": {"weight": t["final.norm"]},
           "head": {"weight": t["embed"]}}
    if mc.step_vectors:
        out["step_vectors"] = {"weight": t["loop.step"]}
    return out


MOGEVIK = Architecture(name=ARCHITECTURE, read_config=read_config, declare_tensors=declare_tensors,
                       bind_tensors=bind_tensors, aliases=("mogevik",))
ModelSupport.add_model(MOGEVIK)
