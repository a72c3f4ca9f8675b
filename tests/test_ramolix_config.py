"""Ramolix without a GPU: the configuration reader and what it refuses, tensor names and shapes, what each layer keeps
between steps, and invariants of the plain implementation's mechanisms."""

import copy
import math

import pytest
import torch

import plain_ramolix as pr
from ramolix_configs import SMALL, SMALL_B, SMALL_C, SMALL_D, STRETCH

F64 = torch.float64


def spec_of(config):
    from llmserve.models.ramolix import RamolixConfig, ramolix_spec

    return ramolix_spec(RamolixConfig.from_dict(config))


def model_of(config, dtype=torch.float32):
    from llmserve.parts.model import Model
    from llmserve.parts.registry import BuildContext

    return Model(spec_of(config), BuildContext(dtype, torch.device("cpu")))


def rnd(*shape, seed=0, scale=1.0):
    return scale * torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


def test_the_registry_finds_the_design_by_its_name():
    from llmserve.config.registry import architecture_of, preset

    assert architecture_of(SMALL).name == "Ramolix"
    for name in ("ramolix-tiny", "ramolix-1b"):
        assert architecture_of(preset(name)).name == "Ramolix"
        spec_of(preset(name))


def test_tensor_names_and_shapes():
    shape = {k: tuple(v.shape) for k, v in model_of(SMALL).param_infos().items()}
    w = 72
    assert shape["embed"] == (151, w) and "head" not in shape and shape["final.norm"] == (w,)
    assert all(shape[f"l{i}.norm1"] == (w,) for i in range(6))
    assert shape["l0.mix.q"] == (36, w) and shape["l0.mix.dkv"] == (40, w) and shape["l0.mix.dkv.norm"] == (40,)
    assert shape["l0.mix.uk"] == (36, 40) and shape["l0.mix.uv"] == (60, 40) and shape["l0.mix.o"] == (w, 60)
    assert shape["l1.mix.in"] == (72 + 72 + 60 + 60 + 6, w) and shape["l1.mix.conv"] == (192, 4) and shape["l1.mix.conv.b"] == (192,)
    assert shape["l1.mix.dt_bias"] == shape["l1.mix.A_log"] == shape["l1.mix.D"] == (6,)
    assert shape["l1.mix.norm"] == (72,) and shape["l1.mix.o"] == (w, 72)
    assert shape["l2.mix.q"] == (96, w) and shape["l2.mix.q.b"] == (96,) and shape["l2.mix.q.norm"] == (96,)
    assert shape["l2.mix.k"] == (48, w) and shape["l2.mix.k.b"] == (48,) and shape["l2.mix.k.norm"] == (48,)
    assert "l2.mix.v" not in shape and shape["l2.mix.o"] == (w, 96)
    assert "l3.mix.dkv" not in shape and "l3.mix.dkv.norm" not in shape and shape["l3.mix.uk"] == (40, 40) and shape["l3.mix.uv"] == (40, 40)
    assert shape["l0.mlp.gate"] == shape["l0.mlp.up"] == (56, w) and shape["l0.mlp.down"] == (w, 56)
    # a layer without a feed-forward has no second norm of its own, and a checkpoint may still hold it
    assert "l4.norm2" not in shape and "l4.mlp.up" not in shape and spec_of(SMALL).unused_tensors == ("l4.norm2",)


def test_what_each_layer_keeps():
    model = model_of(SMALL)
    a, b, c, d, e, f = model.cache_specs()
    assert (a.num_kv_heads, a.head_dim, a.v_heads, a.v_dim, a.window) == (1, 40, 0, 0, None)
    assert d is None and f is None and model.cache_sources() == [None, None, None, 0, None, 0]
    assert (c.num_kv_heads, c.head_dim, c.v_heads, c.v_dim, c.window) == (2, 24, 2, 24, 13)
    assert b.shape == (6 * 12 * 20 + 3 * 192,) and b.dtype == "float32"
    assert e.shape == (6 * 12 * 20 + 3 * (72 + 40),)
    b_specs = model_of(SMALL_B).cache_specs()
    assert b_specs[0].window == 1 and b_specs[2].window is None
    assert b_specs[1].shape == (4 * 7 * 3,)  # one tap: no ring
    assert b_specs[4].shape == (33 * 9 + 51 + 0,) and (33 * 9 + 51) % 4 == 0


def test_slots_are_multiples_of_sixteen_bytes():
    for config in (SMALL, SMALL_B, SMALL_C, SMALL_D):
        for spec in model_of(config).cache_specs():
            assert not hasattr(spec, "shape") or spec.shape[0] % 4 == 0


def test_the_libraries_follow_the_sizes_and_the_dtype():
    names = model_of(SMALL_D, torch.bfloat16).libraries("bfloat16")
    assert {"attention_mfma", "latent_mfma", "state_space", "stream32"} <= set(names) and "attention_gated" not in names
    names = model_of(SMALL_D).libraries("float32")
    assert "attention_mfma" not in names and "state_space" in names
    for config in (SMALL, SMALL_B, SMALL_C, SMALL_D):
        assert model_of(config).graph_safe()


@pytest.mark.parametrize("bad", [
    lambda c: c["layers"][0].update(type="delta"),
    lambda c: c["layers"][0]["mixer"].pop("scale"),
    lambda c: c["layers"][0]["mixer"].update(kv_rank=0),
    lambda c: c["layers"][1]["mixer"].update(groups=4),
    lambda c: c["layers"][1]["mixer"].update(norm_groups=5),
    lambda c: c["layers"][1]["mixer"].update(conv=0),
    lambda c: c["layers"][1]["mixer"].pop("state"),
    lambda c: c["layers"][2]["mixer"].update(heads=3),
    lambda c: c["layers"][2]["mixer"].update(vdim=12),
    lambda c: c["layers"][2]["mixer"].update(mask={"size": 0}),
    lambda c: c["layers"][2]["mixer"]["rot"].update(dims=26),
    lambda c: c["layers"][2]["mixer"]["rot"].update(dims=7),
    lambda c: c["layers"][2]["mixer"]["rot"].update(scaling={"factor": 2.0}),
    lambda c: c["layers"][3]["mixer"].update(kv_from=1),
    lambda c: c["layers"][3]["mixer"].update(kv_from=3),
    lambda c: c["layers"][3]["mixer"].update(kv_from=-1),
    lambda c: c["layers"][3]["mixer"].update(kv_rank=24),
    lambda c: c["layers"][5]["mixer"].update(kv_from=3),
    lambda c: c["layers"][0]["mlp"].update(ff=0),
    lambda c: c["layers"][0]["mlp"].update(kind="moe"),
    lambda c: c["norm"].update(eps=0),
    lambda c: c.pop("vocab"),
])
def test_what_the_reader_refuses(bad):
    from llmserve.config.model_config import ConfigError
    from llmserve.models.ramolix import RamolixConfig

    config = copy.deepcopy(SMALL)
    bad(config)
    with pytest.raises(ConfigError):
        RamolixConfig.from_dict(config)


def test_the_configuration_goes_to_json_and_back():
    from llmserve.models.ramolix import RamolixConfig

    for config in (SMALL, SMALL_B, SMALL_C, SMALL_D):
        cfg = RamolixConfig.from_dict(config)
        assert RamolixConfig.from_dict(cfg.to_dict()) == cfg


def test_the_engine_and_the_plain_frequencies_agree():
    from llmserve.parts.attention_composed import scaled_frequencies

    for base, dims, scaling in ((50.0, 16, STRETCH), (1e5, 12, dict(STRETCH, factor=8.0)), (100.0, 2, None)):
        want = pr.frequencies({"base": base, "dims": dims, "scaling": scaling})
        assert torch.allclose(torch.tensor(scaled_frequencies(base, dims, scaling), dtype=F64), want, rtol=1e-12)
    f = pr.frequencies({"base": 50.0, "dims": 16, "scaling": STRETCH})
    plain = pr.frequencies({"base": 50.0, "dims": 16})
    ratio = plain / f
    assert abs(float(ratio[0]) - 1.0) < 1e-12 and abs(float(ratio[-1]) - 3.0) < 1e-12
    assert any(1.01 < float(r) < 2.99 for r in ratio)  # all three regimes


# ------------------------------------------------------------------------------ the plain mechanisms
def test_gelu_reduces_to_the_library_routine():
    x = rnd(500, scale=3.0)
    assert torch.allclose(pr.gelu_tanh(x), torch.nn.functional.gelu(x, approximate="tanh"), atol=1e-14)


def test_the_recurrence_is_attention_with_decays():
    """y_t = sum_(s <= t) (C_t . B_s) exp(A sum_(s < u <= t) dt_u) dt_s x_s + D x_t, written out."""
    T, H, P, G, N = 17, 4, 3, 2, 5
    x, B, C = rnd(T, H, P, seed=1), rnd(T, G, N, seed=2), rnd(T, G, N, seed=3)
    dt, A, D = rnd(T, H, seed=4).abs(), -rnd(H, seed=5).abs(), rnd(H, seed=6)
    got = pr.state_space(x, B, C, dt, A, D)
    for h in range(H):
        g, L = h // 2, torch.cumsum(dt[:, h] * A[h], 0)
        m = (C[:, g] @ B[:, g].T) * torch.exp(L[:, None] - L[None, :]) * dt[None, :, h]
        want = torch.tril(m) @ x[:, h] + D[h] * x[:, h]
        assert torch.allclose(got[:, h], want, atol=1e-12)


def test_the_normed_parts_have_unit_mean_square_and_the_gate_comes_first():
    y, z = rnd(9, 24, seed=7), rnd(9, 24, seed=8)
    out = pr.gated_group_norm(y, z, torch.ones(24, dtype=F64), 4, 0.0)
    assert torch.allclose((out.view(9, 4, 6) ** 2).mean(-1), torch.ones(9, 4, dtype=F64))
    scaled = pr.gated_group_norm(y * torch.tensor([3.0] * 6 + [1.0] * 18), z, torch.ones(24, dtype=F64), 4, 0.0)
    assert torch.allclose(scaled, out)  # a factor on a whole part is normed away
    assert not torch.allclose(pr.rms(y.view(9, 4, 6), 0.0).view(9, 24) * pr.silu(z), out)


def test_the_convolution_reduces_to_the_library_routine():
    x, w, b = rnd(11, 6, seed=1), rnd(6, 4, seed=2), rnd(6, seed=3)
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(x.T[None], (3, 0)), w[:, None], b, groups=6)[0].T
    assert torch.allclose(pr.causal_conv(x, w, b), want)


def test_a_window_of_one_key_gives_a_token_its_own_projected_key():
    m = {"heads": 4, "kv_heads": 2, "dim": 6, "scale": 0.7, "mask": {"size": 1}, "rot": {"base": 10.0, "dims": 4}}
    h = rnd(8, 10, seed=1)
    t = {"q": rnd(24, 10, seed=2), "k": rnd(12, 10, seed=3), "q.b": rnd(24, seed=4), "k.b": rnd(12, seed=5), "q.norm": rnd(24, seed=6),
         "k.norm": rnd(12, seed=7), "o": torch.eye(24, dtype=F64)}
    raw = (h @ t["k"].T + t["k.b"]).view(8, 2, 6)
    assert torch.allclose(pr.attention(h, t, "", m, 1e-5), raw.repeat_interleave(2, dim=1).reshape(8, 24))


def test_the_latent_mixer_with_its_keys_folded_into_the_query():
    m = {"heads": 3, "dim": 5, "vdim": 4, "kv_rank": 7, "scale": 0.3}
    h = rnd(9, 11, seed=1)
    t = {"q": rnd(15, 11, seed=2), "dkv": rnd(7, 11, seed=3), "dkv.norm": rnd(7, seed=4), "uk": rnd(15, 7, seed=5), "uv": rnd(12, 7, seed=6),
         "o": torch.eye(12, dtype=F64)}
    c = pr.latents(h, t, "", 1e-5)
    out = pr.latent_attention(h, c, t, "", m).view(9, 3, 4)
    for a in range(3):
        folded = (h @ t["q"].T).view(9, 3, 5)[:, a] @ t["uk"].view(3, 5, 7)[a]
        w = torch.softmax((folded @ c.T * 0.3).masked_fill(~pr.visible(9), -math.inf), -1)
        assert torch.allclose(out[:, a], (w @ c) @ t["uv"].view(3, 4, 7)[a].T)


def test_a_layer_without_results_scales_nothing_and_the_factor_counts():
    x, y, w = rnd(4, 6, seed=1), rnd(4, 6, seed=2), rnd(6, seed=3)
    assert torch.allclose(pr.joined(x, 100.0 * y, w, 0.0, 0.5), pr.joined(x, y, w, 0.0, 0.5))
    assert torch.allclose(pr.joined(x, y, w, 0.0, 0.5) - x, 0.25 * (pr.joined(x, y, w, 0.0, 2.0) - x))
