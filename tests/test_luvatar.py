"""Luvatar without a GPU: its configuration, run order, tensor declarations, the random-weights mode, what its mixers
ask of the cache and how the cache manager gives a chunk's pages back, and the plain implementation against other ways
of writing the same formulas."""
import json

import numpy as np
import pytest
import torch

import plain_luvatar as P
from luvatar_models import CONFIG_A, CONFIG_B, CONFIG_C


def test_config_reads_every_size_and_constant():
    from deliverance_amd.config import ConfigError, LuvatarConfig
    from deliverance_amd.config.specs import AttentionSpec, GatedFeedForwardSpec, GatedLinearSpec, LinearSpeedsSpec
    for cfg in (CONFIG_A, CONFIG_B, CONFIG_C):
        mc = LuvatarConfig.from_dict(cfg).to_model_config()
        assert (mc.vocab_size, mc.width, mc.embed_scale) == (cfg["vocab"], cfg["width"], cfg["embedding"]["scale"])
        assert mc.tie_word_embeddings and mc.embed_position.kind == "none" and mc.embed_norm is None
        assert mc.final_norm.kind == "rmsnorm" and mc.final_norm.gain_offset == 0.0 and mc.final_norm.eps == cfg["norm"]["eps"]
        for spec, raw in zip(mc.layers, cfg["layers"]):
            m, a = raw["mixer"], spec.mixer
            assert spec.pre_mixer_norm is None and spec.pre_ff_norm is None and spec.post_mixer_norm.eps == cfg["norm"]["eps"]
            if raw["type"] == "gla":
                assert isinstance(a, GatedLinearSpec)
                assert (a.n_heads, a.head_dim, a.v_head_dim, a.tau, a.decay_rank, a.norm_eps) == \
                    (m["heads"], m["dim"], m["vdim"], m["tau"], m["a_rank"], cfg["norm"]["eps"])
            else:
                assert isinstance(a, AttentionSpec) and a.sink == "learned" and a.out_gate == "sigmoid" and a.window is None
                assert (a.n_heads, a.n_kv_heads, a.head_dim, a.value_dim, a.scale) == \
                    (m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"])
                assert a.chunk == (m["mask"] or {}).get("size") and a.shared_kv == ("kv_from" in m)
                assert not a.qk_norm.whole and a.qk_norm.eps == cfg["norm"]["eps"] and not a.qkv_bias and not a.out_bias
                assert (a.position.dims, a.position.base, a.position.interleaved) == (m["rot"]["dims"], m["rot"]["base"], True)
                sc = m["rot"].get("scaling")
                assert a.position.scaling == (LinearSpeedsSpec(sc["factor"]) if sc else None)
            if raw["mlp"] is None:
                assert spec.feed_forward is None and spec.post_ff_norm is None
            else:
                assert isinstance(spec.feed_forward, GatedFeedForwardSpec) and spec.feed_forward.activation == "silu"
                assert spec.feed_forward.inner == raw["mlp"]["ff"] and spec.post_ff_norm is not None
        assert LuvatarConfig.from_dict(mc.raw).to_model_config() == mc           # what is written out reads back the same
    # what is missing is named, all of it at once
    broken = json.loads(json.dumps(CONFIG_A))
    del broken["norm"]["eps"], broken["embedding"]["scale"], broken["layers"][1]["mixer"]["tau"], broken["layers"][0]["mixer"]["mask"]["size"]
    del broken["layers"][0]["mlp"]["ff"], broken["layers"][2]["mixer"]["rot"]["scaling"]["factor"], broken["layers"][3]["mixer"]["vdim"]
    with pytest.raises(ConfigError) as e:
        LuvatarConfig.from_dict(broken)
    for key in ("norm.eps", "embedding.scale", "layers[1].mixer.tau", "layers[0].mixer.mask.size", "layers[0].mlp.ff",
                "layers[2].mixer.rot.scaling.factor", "layers[3].mixer.vdim"):
        assert key in str(e.value)
    for change, match in ((lambda c: c["layers"][0].update(type="retention"), "retention"),
                          (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "rot.dims"),
                          (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "key heads"),
                          (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "moe"),
                          (lambda c: c["layers"][2]["mixer"].update(kv_from=3), "kv_from"),
                          (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "kv_from"),
                          (lambda c: c["layers"][2]["mixer"].update(dim=8, rot={"base": 10000.0, "dims": 8}), "differ"),
                          (lambda c: c["layers"][2]["mixer"]["rot"].update(base=500.0), "differ"),
                          (lambda c: c["layers"][1]["mixer"].update(tau=0.0), "tau")):
        other = json.loads(json.dumps(CONFIG_A))
        change(other)
        with pytest.raises(ConfigError, match=match):
            LuvatarConfig.from_dict(other)
    chain = json.loads(json.dumps(CONFIG_B))
    chain["layers"][3]["mixer"]["kv_from"] = 2
    with pytest.raises(ConfigError, match="of its own"):
        LuvatarConfig.from_dict(chain)


def test_a_layer_on_anothers_keys_reads_that_layers_slot():
    from deliverance_amd.config import LuvatarConfig
    mc = LuvatarConfig.from_dict(CONFIG_A).to_model_config()
    assert [(c.layer, c.cache, c.write) for c in mc.schedule] == [(0, 0, True), (1, 1, True), (2, 0, False), (3, 3, True)]
    mc = LuvatarConfig.from_dict(CONFIG_B).to_model_config()
    assert [(c.layer, c.cache, c.write) for c in mc.schedule] == [(0, 0, True), (1, 1, True), (2, 1, False), (3, 1, False)]


def test_tensors_and_what_the_mixers_keep(tmp_path):
    from deliverance_amd import models  # noqa: F401
    from deliverance_amd.parts import KVNeed, StateNeed
    from deliverance_amd.random_model import random_model
    from deliverance_amd.registry import ModelSupport
    from deliverance_amd.weights.loader import load_declared
    arch = ModelSupport.detect(CONFIG_A)
    assert arch.name == "Luvatar"
    mc = arch.read_config(CONFIG_A)
    names = {d.name: tuple(d.shape) for d in arch.declare_tensors(mc)}
    E = CONFIG_A["width"]
    assert names["embed"] == (CONFIG_A["vocab"], E) and "head" not in names and names["final.norm"] == (E,)
    assert names["l0.mix.k"] == (2 * 16, E) and names["l0.mix.v"] == (2 * 8, E) and names["l0.mix.g"] == (4 * 8, E)
    assert names["l0.mix.q.norm"] == (16,) and names["l0.mix.k.norm"] == (16,) and names["l0.mix.sink"] == (4,)
    assert names["l1.mix.a1"] == (8, E) and names["l1.mix.a2"] == (3 * 16, 8) and names["l1.mix.a2.b"] == (3 * 16,)
    assert names["l1.mix.norm"] == (24,) and names["l1.mix.o"] == (E, 3 * 24) and "l1.norm2" not in names
    assert {"l2.mix.q", "l2.mix.q.norm", "l2.mix.g", "l2.mix.sink", "l2.mix.o"} <= set(names)
    assert not {"l2.mix.k", "l2.mix.v", "l2.mix.k.norm"} & set(names)
    # a config.json without the rank leaves it to the checkpoint
    open_cfg = json.loads(json.dumps(CONFIG_A))
    for L in open_cfg["layers"]:
        L["mixer"].pop("a_rank", None)
    assert {d.name: tuple(d.shape) for d in arch.declare_tensors(arch.read_config(open_cfg))}["l1.mix.a1"] == (-1, E)
    random_model(str(tmp_path), CONFIG_A, 3)
    (tmp_path / "config.json").write_text(json.dumps(open_cfg))
    mc = arch.read_config(open_cfg)
    t = load_declared(str(tmp_path), arch.declare_tensors(mc))
    from deliverance_amd.kernels import build
    if not build.is_built():
        pytest.skip("the kernel libraries are not built")
    from deliverance_amd.models.causal_lm import CausalLM
    model = CausalLM(mc, arch.bind_tensors(mc, t), torch.float32, "cpu")
    needs = model.cache_needs()
    assert sorted(needs) == [0, 1, 3]
    assert needs[0] == KVNeed(2, 16, 50, 8)             # chunks of 20 and of 50 read it: what either sees lies within 50 keys
    assert needs[1] == StateNeed(3 * 24 * 16) and needs[3] == StateNeed(2 * 16 * 32)
    mc = arch.read_config(CONFIG_B)
    random_model(str(tmp_path / "b"), CONFIG_B, 4)
    model = CausalLM(mc, arch.bind_tensors(mc, load_declared(str(tmp_path / "b"), arch.declare_tensors(mc))), torch.float32, "cpu")
    assert model.cache_needs()[1] == KVNeed(1, 12, None, 20)         # one of its readers sees every earlier key


def test_needs_of_two_masks_on_one_slot():
    from deliverance_amd.parts import KVNeed
    n = lambda **k: KVNeed(2, 16, v_head_dim=8, **k)
    assert n(chunk=20).joined(n(chunk=20)) == n(chunk=20)
    assert n(chunk=20).joined(n(chunk=50)) == n(window=50) == n(chunk=50).joined(n(chunk=20))
    assert n(chunk=20).joined(n(window=7)) == n(window=20)
    assert n(chunk=20).joined(n()) == n() and n(window=9, keep_first=3).joined(n(window=9)) == n(window=9, keep_first=3)
    with pytest.raises(ValueError):
        n(chunk=20).joined(KVNeed(1, 16, v_head_dim=8, chunk=20))


def test_a_chunks_pages_go_back_when_the_next_chunk_starts():
    """Pages of 16, chunks of 40: while positions 40 .. 79 come, the page that holds 32 .. 47 stays (it holds the chunk's
    first keys) and the two before it go; a request's next chunk starts at 80, a page's edge."""
    from deliverance_amd.cache.manager import CacheManager, KVGroupSpec
    m = CacheManager([KVGroupSpec((0,), 1, 16, chunk=40)], 16, [6])
    m.open("a")
    m.extend("a", 39)
    assert m.commit("a") == [] and [p >= 0 for p in m.table("a", 0)] == [True] * 3       # the next one, 39, still sees 0
    m.extend("a", 1)
    released = m.commit("a")                                                             # the next one, 40, sees 40 only
    assert len(released) == 2 and [p >= 0 for p in m.table("a", 0)] == [False, False, True]
    m.extend("a", 39)
    assert m.commit("a") == [] and [p >= 0 for p in m.table("a", 0)] == [False, False, True, True, True]
    m.extend("a", 1)
    assert len(m.commit("a")) == 3 and not any(p >= 0 for p in m.table("a", 0))
    m.check()
    m.extend("a", 41)                                                                    # a portion across a chunk's edge
    assert sum(p >= 0 for p in m.table("a", 0)) == 3
    m.commit("a")                                                                        # 121 are held, the next sees from 120 on
    assert [p >= 0 for p in m.table("a", 0)][-1] and sum(p >= 0 for p in m.table("a", 0)) == 1
    m.close("a")
    m.check()
    assert m.pools[0].n_free == 6


def test_the_plain_model_written_another_way():
    """Gated linear attention as a sum over earlier tokens with products of the decays between; attention chunk by
    chunk as full attention over each chunk's rows alone; the extra term as one more key whose value is zero; slowed
    speeds as positions closer together."""
    rng = np.random.default_rng(0)
    T, E = 23, 16
    m = {"heads": 2, "dim": 8, "vdim": 4, "tau": 2.0}
    W = {"mix.q": rng.normal(size=(16, E)), "mix.k": rng.normal(size=(16, E)), "mix.v": rng.normal(size=(8, E)),
         "mix.g": rng.normal(size=(8, E)), "mix.o": rng.normal(size=(E, 8)), "mix.a1": rng.normal(size=(3, E)),
         "mix.a2": rng.normal(size=(16, 3)), "mix.a2.b": rng.normal(size=16), "mix.norm": rng.normal(size=4)}
    h = rng.normal(size=(T, E))
    got = P.gated_linear(W, "", m, h, 1e-5)
    q, k = (h @ W["mix.q"].T).reshape(T, 2, 8) / np.sqrt(8.0), (h @ W["mix.k"].T).reshape(T, 2, 8)
    v = (h @ W["mix.v"].T).reshape(T, 2, 4)
    a = (1.0 / (1.0 + np.exp(-(h @ W["mix.a1"].T @ W["mix.a2"].T + W["mix.a2.b"])))) ** 0.5
    a = a.reshape(T, 2, 8)
    o = np.zeros((T, 2, 4))
    for t in range(T):
        for s in range(t + 1):
            between = np.prod(a[s + 1:t + 1], axis=0)
            o[t] += (q[t] * between * k[s]).sum(-1)[:, None] * v[s]
    o = o / np.sqrt((o ** 2).mean(-1, keepdims=True) + 1e-5) * W["mix.norm"]
    gate = h @ W["mix.g"].T
    want = (o.reshape(T, 8) * gate / (1.0 + np.exp(-gate))) @ W["mix.o"].T
    assert np.abs(got - want).max() <= 1e-9 * np.abs(want).max()
    # attention, chunk by chunk
    m = {"heads": 4, "kv_heads": 2, "dim": 8, "vdim": 4, "scale": 0.3, "mask": {"size": 7}, "rot": {"base": 100.0, "dims": 4, "scaling": {"factor": 2.0}}}
    W = {"mix.q": rng.normal(size=(32, E)), "mix.k": rng.normal(size=(16, E)), "mix.v": rng.normal(size=(8, E)), "mix.g": rng.normal(size=(16, E)),
         "mix.o": rng.normal(size=(E, 16)), "mix.sink": rng.normal(size=4), "mix.q.norm": rng.normal(size=8), "mix.k.norm": rng.normal(size=8)}
    kv = P.keys_and_values(W, "", m, h, 1e-5)
    got = P.attention(W, "", m, h, 1e-5, kv)
    q = P.turn_neighbours(P.rms_scaled((h @ W["mix.q"].T).reshape(T, 4, 8), W["mix.q.norm"], 1e-5), np.arange(T), m["rot"])
    out = np.zeros((T, 4, 4))
    for lo in range(0, T, 7):
        for t in range(lo, min(lo + 7, T)):
            for hd in range(4):
                keys, vals = kv[0][lo:t + 1, hd // 2], kv[1][lo:t + 1, hd // 2]
                s = np.concatenate([keys @ q[t, hd] * 0.3, [W["mix.sink"][hd]]])
                w = np.exp(s - s.max())
                out[t, hd] = (w / w.sum())[:-1] @ vals
    want = (out.reshape(T, 16) / (1.0 + np.exp(-(h @ W["mix.g"].T)))) @ W["mix.o"].T
    assert np.abs(got - want).max() <= 1e-9 * np.abs(want).max()
    v = rng.normal(size=(5, 3, 8))
    places = np.array([0, 3, 8, 100, 41])
    half = P.turn_neighbours(v, places, {"base": 50.0, "dims": 6, "scaling": {"factor": 4.0}})
    assert np.abs(half - P.turn_neighbours(v, places / 4.0, {"base": 50.0, "dims": 6})).max() <= 1e-12
    assert np.abs(half[..., 6:] - v[..., 6:]).max() == 0.0


def test_the_engines_speeds_are_the_plain_ones():
    from deliverance_amd.config.specs import LinearSpeedsSpec, RotarySpec
    from deliverance_amd.parts import build_position
    for dims, base, factor in ((16, 5e4, 3.0), (32, 10000.0, None), (8, 100.0, 1.0), (24, 500.0, 0.25)):
        part = build_position(RotarySpec("rotary", dims, base, True, None if factor is None else LinearSpeedsSpec(factor)), {}, torch.float32, "cpu")
        r = {"base": base, "dims": dims}
        if factor is not None:
            r["scaling"] = {"factor": factor}
        assert np.abs(part.speeds.numpy() - P.pair_speeds(r)).max() <= 1e-15 and part.magnitude == 1.0
