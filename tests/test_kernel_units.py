"""The kernel units: every entry point that the engine calls is found in a unit, what a unit needs comes before it, and
the units that a model names for its first call exist.  Compiling: only what is missing of what is asked for."""
import os

import pytest
import torch

import helpers


def test_every_entry_point_has_a_unit():
    from deliverance_amd.kernels import build, ops
    found = build.entry_points()
    names = set(build.units())
    for name in ops._ARGTYPES:
        assert found.get(name) in names, f"{name} is in no unit"
    assert found["da_last_error"] == build.BASE_UNIT
    assert found["da_attn_decode_rel"] == "attn_decode_rel" and found["da_attn_decode"] == "attn_decode"
    assert set(build.NEEDS) <= names and {n for ns in build.NEEDS.values() for n in ns} <= names
    assert set(build.INCLUDES) <= names and set(build.EXTRA_FLAGS) <= names


def test_what_a_unit_needs_comes_first():
    from deliverance_amd.kernels import build
    order = build.with_needs(["run_step", "gla"])
    assert order[0] == build.BASE_UNIT and len(order) == len(set(order))
    assert order.index("gemm_wide") < order.index("gemm_mfma") < order.index("run_step") and "gla" in order
    assert build.with_needs([build.BASE_UNIT]) == [build.BASE_UNIT]


def test_only_what_is_asked_for_and_missing_is_compiled(tmp_path, monkeypatch):
    from deliverance_amd.kernels import build
    done = []

    def compiled(hipcc, out_dir, todo, verbose):
        for u in todo:
            done.append(u)
            with open(os.path.join(out_dir, f"libda_{u}.so"), "w"):
                pass
    monkeypatch.setattr(build, "_build_dirs", lambda: (str(tmp_path / "a"), str(tmp_path / "b")))
    monkeypatch.setattr(build, "_build_locked", compiled)
    monkeypatch.setattr(build, "_find_hipcc", lambda: "hipcc")
    build.build(only=["gla"])
    assert sorted(done) == sorted(["gla", build.BASE_UNIT])
    build.build(only=["gla", "attn_window"])
    assert sorted(done) == sorted(["gla", build.BASE_UNIT, "attn_window"])
    build.build(only=["gla"])
    assert len(done) == 3 and "moe" in build.missing() and build.missing(["gla"]) == []
    build.build(force=True, only=["gla"])
    assert sorted(done[3:]) == sorted(["gla", build.BASE_UNIT])
    monkeypatch.setattr(build, "_find_hipcc", lambda: None)
    with pytest.raises(build.KernelLibraryError, match="hipcc was not found"):
        build.build(only=["moe"])


def test_models_name_units_that_exist(tmp_path):
    from deliverance_amd.kernels import build
    from deliverance_amd.models.causal_lm import load_model
    from deliverance_amd.random_model import random_model
    from luvatar_models import CONFIG_A
    from mogevik_models import CONFIG_D, CONFIG_E
    from pafolorn_models import CONFIG_F
    from pedatar_models import CONFIG_P
    from salivik_models import CONFIG_S
    from virudra_models import CONFIG_X
    names = set(build.units())
    of = {}
    for key, cfg in (("gpt2", helpers.CONFIG_A), ("virudra", CONFIG_X), ("pedatar", CONFIG_P), ("pafolorn", CONFIG_F),
                     ("salivik", CONFIG_S), ("luvatar", CONFIG_A), ("mogevik", CONFIG_D), ("mogevik_plain", CONFIG_E)):
        folder = str(tmp_path / key)
        random_model(folder, cfg, 1)
        for dtype in (torch.bfloat16, torch.float32):
            of[key, dtype] = set(load_model(folder, dtype, "cpu").kernel_units())
            assert of[key, dtype] <= names, f"{key}: {of[key, dtype] - names}"
    lu = of["luvatar", torch.bfloat16]
    assert {"gla", "attn_window", "attn_prepare"} <= lu and not lu & {"moe", "ssm", "retention", "attn_latent", "attn_prefill", "gemm_ref"}
    assert "gla" not in of["gpt2", torch.bfloat16] and "gemm_mfma" not in of["luvatar", torch.float32]
    mo = of["mogevik", torch.bfloat16]
    assert {"rglru", "moe", "attn_window", "elementwise"} <= mo and not mo & {"ssm", "gla", "attn_prepare", "norm_rms", "gemm_ref", "attn_latent"}
    assert {"rglru", "ssm"} <= of["mogevik_plain", torch.bfloat16] and {"rglru", "ssm", "attn_rel"} <= of["mogevik", torch.float32]
    from deliverance_amd.kernels import ops
    if build.is_built():
        assert all(bool(ops._lib().da_rglru_serve_takes(n)) == ops.rglru_block_fits(n) for n in range(1, 300))
