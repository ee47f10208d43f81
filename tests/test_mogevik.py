"""Mogevik without a GPU: its configuration, run order, tensor declarations, the random-weights mode, what its mixers ask
of the cache, and the plain implementation against other ways of writing the same formulas."""
import json

import numpy as np
import pytest
import torch

import plain_mogevik as P
from mogevik_models import CONFIG_D, CONFIG_E, CONFIG_F


def test_config_reads_every_size_and_constant():
    from deliverance_amd.config import ConfigError, MogevikConfig
    from deliverance_amd.config.specs import AttentionSpec, ExpertsFeedForwardSpec, RealGatedRecurrenceSpec
    for cfg in (CONFIG_D, CONFIG_E, CONFIG_F):
        mc = MogevikConfig.from_dict(cfg).to_model_config()
        assert (mc.vocab_size, mc.width, mc.embed_scale) == (cfg["vocab"], cfg["width"], cfg["embedding"]["scale"])
        assert mc.tie_word_embeddings and mc.embed_position.kind == "none"
        assert mc.final_norm.kind == "layernorm" and not mc.final_norm.bias and mc.final_norm.eps == cfg["norm"]["eps"]
        assert mc.step_vectors == ((cfg["loop"] or {}).get("times") or 0)
        for spec, raw in zip(mc.layers, cfg["layers"]):
            m, a, f = raw["mixer"], spec.mixer, spec.feed_forward
            assert spec.pre_mixer_norm == mc.final_norm and spec.pre_ff_norm is None and spec.parallel == (raw["mlp"] is not None)
            if raw["type"] == "rglru":
                assert isinstance(a, RealGatedRecurrenceSpec)
                assert (a.channels, a.blocks, a.conv_taps, a.decay_strength) == (m["width"], m["blocks"], m["conv"], 8.0)
            else:
                assert isinstance(a, AttentionSpec) and a.out_gate == "sigmoid" and a.sink is None and a.position is None
                assert (a.n_heads, a.n_kv_heads, a.head_dim, a.value_dim, a.scale) == \
                    (m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"])
                assert a.window == (m["mask"] or {}).get("size") and a.qkv_bias and not a.out_bias
                assert np.abs(np.array(a.distance_slopes) - P.head_slopes(m["heads"])).max() == 0.0
            if raw["mlp"] is None:
                assert f is None
                continue
            ro = raw["mlp"]["router"]
            assert isinstance(f, ExpertsFeedForwardSpec) and f.activation == "silu" and f.router == "softmax_all"
            assert (f.inner, f.n_experts, f.top, f.identity) == (raw["mlp"]["expert"]["ff"], ro["experts"], ro["top"], ro.get("identity", 0))
            assert (f.groups, f.groups_kept) == ((ro["groups"]["count"], ro["groups"]["keep"]) if ro.get("groups") else (0, 0))
            assert f.shared_inner == (raw["mlp"]["shared"] or {}).get("ff", 0)
        assert MogevikConfig.from_dict(mc.raw).to_model_config() == mc           # what is written out reads back the same
    # what is missing is named, all of it at once
    broken = json.loads(json.dumps(CONFIG_D))
    del broken["norm"]["eps"], broken["embedding"]["scale"], broken["loop"]["times"], broken["layers"][0]["mixer"]["blocks"]
    del broken["layers"][0]["mlp"]["router"]["groups"]["keep"], broken["layers"][1]["mixer"]["mask"]["size"]
    del broken["layers"][1]["mlp"]["shared"]["ff"], broken["layers"][3]["mixer"]["vdim"], broken["layers"][3]["mlp"]["expert"]
    with pytest.raises(ConfigError) as e:
        MogevikConfig.from_dict(broken)
    for key in ("norm.eps", "embedding.scale", "loop.times", "layers[0].mixer.blocks", "layers[0].mlp.router.groups.keep",
                "layers[1].mixer.mask.size", "layers[1].mlp.shared.ff", "layers[3].mixer.vdim", "layers[3].mlp.expert"):
        assert key in str(e.value)
    for change, match in ((lambda c: c["layers"][0].update(type="gla"), "gla"),
                          (lambda c: c["layers"][0]["mixer"].update(blocks=5), "equal blocks"),
                          (lambda c: c["layers"][1]["mixer"].update(kv_heads=3), "key heads"),
                          (lambda c: c["layers"][1]["mlp"].update(kind="dense"), "dense"),
                          (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=2), "equal groups"),
                          (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=4), "equal groups"),
                          (lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "can be chosen"),
                          (lambda c: c["layers"][1]["mlp"]["router"].update(top=5), "can be chosen"),
                          (lambda c: c["layers"][0]["mixer"].update(conv=0), "conv"),
                          (lambda c: c["loop"].update(stop=9), "loop")):
        other = json.loads(json.dumps(CONFIG_D))
        change(other)
        with pytest.raises(ConfigError, match=match):
            MogevikConfig.from_dict(other)


def test_the_loops_passes_have_slots_and_additions_of_their_own():
    from deliverance_amd.config import MogevikConfig
    order = lambda c: [(x.layer, x.cache, x.add_input, x.add_step) for x in MogevikConfig.from_dict(c).to_model_config().schedule]
    assert order(CONFIG_D) == [(0, 0, False, None), (1, 1, False, 0), (2, 2, False, None), (1, 3, True, 1), (2, 4, False, None),
                               (1, 5, True, 2), (2, 6, False, None), (3, 7, False, None)]
    assert order(CONFIG_E) == [(0, 0, False, None), (1, 1, False, None), (2, 2, False, None)]
    assert order(CONFIG_F) == [(0, 0, False, 0), (1, 1, False, None), (2, 2, False, None),
                               (0, 3, True, 1), (1, 4, False, None), (2, 5, False, None)]


def test_tensors_and_what_the_mixers_keep(tmp_path):
    from deliverance_amd import models  # noqa: F401
    from deliverance_amd.kernels import build
    from deliverance_amd.parts import KVNeed, StateNeed
    from deliverance_amd.random_model import random_model
    from deliverance_amd.registry import ModelSupport
    from deliverance_amd.weights.loader import load_declared
    arch = ModelSupport.detect(CONFIG_D)
    assert arch.name == "Mogevik"
    mc = arch.read_config(CONFIG_D)
    names = {d.name: tuple(d.shape) for d in arch.declare_tensors(mc)}
    E = CONFIG_D["width"]
    assert names["embed"] == (CONFIG_D["vocab"], E) and names["loop.step"] == (3, E) and names["final.norm"] == (E,) and "head" not in names
    assert names["l0.mix.y"] == (48, E) == names["l0.mix.x"] and names["l0.mix.y.b"] == (48,) and names["l0.mix.conv"] == (48, 4)
    assert names["l0.mix.ra"] == (3, 16, 16) and names["l0.mix.ri.b"] == (3, 16) and names["l0.mix.lam"] == (48,) and names["l0.mix.o"] == (E, 48)
    assert names["l1.mix.v"] == (2 * 24, E) and names["l1.mix.v.b"] == (48,) and names["l1.mix.g"] == (4 * 24, E) and "l1.mix.g.b" not in names
    assert names["l0.mlp.router"] == (9, E) and names["l0.mlp.correction"] == (9,) and names["l0.mlp.shared.sg"] == (1, E)
    assert names["l0.mlp.e6.down"] == (E, 24) and "l0.mlp.e7.gate" not in names and "l3.mlp.shared.gate" not in names
    assert not any(n.startswith("l2.mlp") for n in names)
    random_model(str(tmp_path), CONFIG_D, 3)
    if not build.is_built():
        pytest.skip("the kernel libraries are not built")
    from deliverance_amd.models.causal_lm import CausalLM
    model = CausalLM(mc, arch.bind_tensors(mc, load_declared(str(tmp_path), arch.declare_tensors(mc))), torch.float32, "cpu")
    needs = model.cache_needs()
    assert needs == {0: StateNeed(4 * 48), 1: KVNeed(2, 16, 20, 24), 2: StateNeed(2 * 96), 3: KVNeed(2, 16, 20, 24),
                     4: StateNeed(2 * 96), 5: KVNeed(2, 16, 20, 24), 6: StateNeed(2 * 96), 7: KVNeed(6, 32, 45)}
    # the constants that are worked out once
    _, W = P.read_model_folder(str(tmp_path))
    rate = model.blocks[0].mixer.rate.double().numpy()
    assert np.abs(rate + 8.0 * P.softplus(W["l0.mix.lam"])).max() <= 1e-6 * np.abs(rate).max()
    assert np.abs(model.blocks[1].mixer.slopes.double().numpy() - [2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8]).max() == 0.0


def test_parts_side_by_side_take_one_norm():
    from deliverance_amd.config.specs import GatedFeedForwardSpec, LayerSpec, NormSpec, RealGatedRecurrenceSpec
    from deliverance_amd.parts import Block
    norm = NormSpec("layernorm", 8, 1e-5, bias=False)
    ff = GatedFeedForwardSpec("gated", 8, 16, "silu")
    mixer = RealGatedRecurrenceSpec("real_gated_recurrence", 8, 8, 1, 2, 8.0)
    params = {k: {"weight": torch.ones(8)} for k in ("pre_mixer_norm", "pre_ff_norm", "post_mixer_norm")}
    for bad in (dict(pre_ff_norm=norm), dict(post_mixer_norm=norm), dict(residual_multiplier=0.5), dict(feed_forward=None)):
        spec = LayerSpec(**{**dict(mixer=mixer, feed_forward=ff, pre_mixer_norm=norm, parallel=True), **bad})
        with pytest.raises(ValueError, match="side by side"):
            Block(spec, params, torch.float32, "cpu")


def test_the_plain_recurrence_written_another_way():
    """The state as a sum over earlier tokens with the decays between; the filter as a sum over pairs; each block's square
    matrices as one block-diagonal matrix; a decay far below one and one near it."""
    rng = np.random.default_rng(0)
    T, E, C, B, K = 19, 10, 12, 3, 4
    n = C // B
    W = {"mix.y": rng.normal(size=(C, E)), "mix.y.b": rng.normal(size=C), "mix.x": rng.normal(size=(C, E)), "mix.x.b": rng.normal(size=C),
         "mix.conv": rng.normal(size=(C, K)), "mix.conv.b": rng.normal(size=C), "mix.ra": rng.normal(size=(B, n, n)),
         "mix.ra.b": rng.normal(size=(B, n)), "mix.ri": rng.normal(size=(B, n, n)), "mix.ri.b": rng.normal(size=(B, n)),
         "mix.lam": np.linspace(-9.0, 4.0, C), "mix.o": rng.normal(size=(E, C))}
    h = rng.normal(size=(T, E))
    got = P.recurrent_block(W, "", h)
    x = h @ W["mix.x"].T + W["mix.x.b"]
    u = np.array([[W["mix.conv.b"][c] + sum(W["mix.conv"][c, K - 1 - (t - s)] * x[s, c] for s in range(max(0, t - K + 1), t + 1))
                   for c in range(C)] for t in range(T)])
    wide = {k: np.zeros((C, C)) for k in ("ra", "ri")}
    for b in range(B):
        for k in wide:
            wide[k][b * n:(b + 1) * n, b * n:(b + 1) * n] = W["mix." + k][b]
    r, i = (1.0 / (1.0 + np.exp(-(u @ wide[k].T + W[f"mix.{k}.b"].reshape(-1)))) for k in ("ra", "ri"))
    a = np.exp(-8.0 * r * np.log1p(np.exp(W["mix.lam"])))
    S = np.array([sum(np.prod(a[s + 1:t + 1], axis=0) * np.sqrt(1.0 - a[s] ** 2) * i[s] * u[s] for s in range(t + 1)) for t in range(T)])
    y = h @ W["mix.y"].T + W["mix.y.b"]
    y = 0.5 * y * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (y + 0.044715 * y * y * y)))
    want = (S * y) @ W["mix.o"].T
    assert np.abs(got - want).max() <= 1e-9 * np.abs(want).max()


def test_the_plain_attention_written_another_way():
    rng = np.random.default_rng(1)
    T, E, m = 17, 9, {"heads": 6, "kv_heads": 2, "dim": 4, "vdim": 5, "scale": 0.6, "mask": {"size": 5}}
    W = {"mix.q": rng.normal(size=(24, E)), "mix.k": rng.normal(size=(8, E)), "mix.v": rng.normal(size=(10, E)), "mix.q.b": rng.normal(size=24),
         "mix.k.b": rng.normal(size=8), "mix.v.b": rng.normal(size=10), "mix.g": rng.normal(size=(30, E)), "mix.o": rng.normal(size=(E, 30))}
    h = rng.normal(size=(T, E))
    got = P.attention(W, "", m, h)
    out = np.zeros((T, 6, 5))
    for hd in range(6):
        row = lambda k, d, j: W[f"mix.{k}"][j * d:(j + 1) * d]
        for t in range(T):
            q = row("q", 4, hd) @ h[t] + W["mix.q.b"][hd * 4:hd * 4 + 4]
            near = range(max(0, t - 4), t + 1)
            e = np.array([np.exp(0.6 * q @ (row("k", 4, hd // 3) @ h[j] + W["mix.k.b"][hd // 3 * 4:][:4]) - (t - j) / 2 ** (8 * (hd + 1) / 6)) for j in near])
            v = np.array([row("v", 5, hd // 3) @ h[j] + W["mix.v.b"][hd // 3 * 5:][:5] for j in near])
            out[t, hd] = (e / e.sum()) @ v
    want = (out.reshape(T, 30) / (1.0 + np.exp(-(h @ W["mix.g"].T)))) @ W["mix.o"].T
    assert np.abs(got - want).max() <= 1e-9 * np.abs(want).max()


def test_the_plain_choice_on_cases_made_by_hand():
    z = np.log(np.array([[0.30, 0.05, 0.20, 0.25, 0.15, 0.05]]))
    none = np.zeros(6)
    ids, w = P.choose(z, none, 2)
    assert ids.tolist() == [[0, 3]] and np.abs(w - [[0.30 / 0.55, 0.25 / 0.55]]).max() < 1e-12
    # the correction decides and does not weigh
    ids, w = P.choose(z, np.array([0.0, 0.5, 0.0, 0.0, 0.0, 0.0]), 2)
    assert ids.tolist() == [[1, 0]] and np.abs(w - [[0.05 / 0.35, 0.30 / 0.35]]).max() < 1e-12
    # three groups of two: {0, 1} and {2, 3} are kept; one of one keeps its small entry too
    ids, _ = P.choose(z, none, 3, {"count": 3, "keep": 2})
    assert ids.tolist() == [[0, 3, 2]]
    ids, _ = P.choose(z, none, 2, {"count": 3, "keep": 1})
    assert ids.tolist() == [[0, 1]]
    # choice scores below zero: what is not kept must not win with a zero
    ids, _ = P.choose(z, np.full(6, -1.0), 2, {"count": 2, "keep": 1})
    assert ids.tolist() == [[0, 2]]
    assert P.nearly_as_good((np.exp(z))[0], [0, 3], None, 0.0) and not P.nearly_as_good(np.exp(z)[0], [0, 2], None, 0.04)
    assert P.nearly_as_good(np.exp(z)[0], [0, 2], None, 0.06) and not P.nearly_as_good(np.exp(z)[0], [0, 3], {"count": 3, "keep": 1}, 0.04)
    assert P.nearly_as_good(np.exp(z)[0], [3, 2], {"count": 3, "keep": 1}, 0.06)
