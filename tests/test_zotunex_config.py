"""Zotunex without a GPU: the configuration reader and what it refuses, tensor names and shapes, what each layer keeps
between steps, the frequencies, and invariants of the plain implementation's mechanisms."""

import copy
import math

import pytest
import torch

import plain_zotunex as pz
from zotunex_configs import SMALL, SMALL_B, SMALL_C, SMALL_D

F64 = torch.float64


def spec_of(config):
    from llmserve.models.zotunex import ZotunexConfig, zotunex_spec

    return zotunex_spec(ZotunexConfig.from_dict(config))


def model_of(config, dtype=torch.float32):
    from llmserve.parts.model import Model
    from llmserve.parts.registry import BuildContext

    return Model(spec_of(config), BuildContext(dtype, torch.device("cpu")))


def rnd(*shape, seed=0, scale=1.0):
    return scale * torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


def test_the_registry_finds_the_design_by_its_name():
    from llmserve.config.registry import architecture_of, preset

    assert architecture_of(SMALL).name == "Zotunex"
    for name in ("zotunex-tiny", "zotunex-1b"):
        assert architecture_of(preset(name)).name == "Zotunex"
        spec_of(preset(name))


def test_tensor_names_and_shapes():
    shape = {k: tuple(v.shape) for k, v in model_of(SMALL).param_infos().items()}
    w = 72
    assert shape["embed"] == (151, w) and shape["head"] == (151, w) and shape["final.norm"] == ()
    for i in range(4):
        assert shape[f"l{i}.norm1"] == () and shape[f"l{i}.norm2"] == ()
    assert shape["l0.mix.q"] == (96, w) and shape["l0.mix.k"] == (48, w) and "l0.mix.v" not in shape
    assert shape["l0.mix.q.norm"] == (24,) and shape["l0.mix.k.norm"] == (24,) and shape["l0.mix.temp"] == (4,)
    assert shape["l0.mix.g"] == (4, w) and shape["l0.mix.o"] == (w, 96)
    assert shape["l0.mlp.up"] == (56, w) and shape["l0.mlp.down"] == (w, 56) and "l0.mlp.gate" not in shape
    assert shape["l1.mix.q"] == (60, w) and shape["l1.mix.dkv"] == (48, w) and shape["l1.mix.dkv.norm"] == (40,)
    assert shape["l1.mix.uk"] == (36, 40) and shape["l1.mix.uv"] == (60, 40) and shape["l1.mix.sink"] == (3,)
    assert shape["l1.mix.g"] == (3, w) and shape["l1.mix.o"] == (w, 60)
    assert not any(name.startswith("l1.mix.dq") or name == "l1.mix.uq" for name in shape)
    assert shape["l1.mlp.router"] == (6, w) and shape["l1.mlp.correction"] == (6,)
    assert shape["l1.mlp.e5.gate"] == (24, w) and shape["l1.mlp.e5.down"] == (w, 24) and "l1.mlp.e6.up" not in shape
    assert shape["l1.mlp.shared.gate"] == (40, w) and shape["l1.mlp.shared.down"] == (w, 40)
    assert "l1.mlp.shared.sg" not in shape and "l1.mlp.router.b" not in shape
    # a layer without a feed-forward has no second norm of its own, and a checkpoint may still hold it
    names_b = model_of(SMALL_B).param_infos()
    assert "l0.norm2" not in names_b and "l0.mlp.up" not in names_b and "l1.mlp.shared.gate" not in names_b
    assert {"l0.norm2", "l2.norm2"} == set(spec_of(SMALL_B).unused_tensors)


def test_what_each_layer_keeps():
    a, b, c, d = model_of(SMALL).cache_specs()
    assert (a.num_kv_heads, a.head_dim, a.v_heads, a.v_dim, a.window) == (2, 24, 2, 24, None)
    assert (b.num_kv_heads, b.head_dim, b.v_heads, b.v_dim, b.window) == (1, 48, 0, 0, None)
    assert a == c and d.head_dim == 44


def test_the_libraries_follow_the_sizes_and_the_dtype():
    assert "attention_gated" in model_of(SMALL_D, torch.bfloat16).libraries("bfloat16")
    assert "attention_gated" not in model_of(SMALL_D).libraries("float32")
    for config in (SMALL, SMALL_B, SMALL_C, SMALL_D):
        assert model_of(config).graph_safe()


@pytest.mark.parametrize("bad", [
    lambda c: c["layers"][0].update(type="delta"),
    lambda c: c["layers"][0]["mixer"].update(heads=3),
    lambda c: c["layers"][0]["mixer"].update(vdim=12),
    lambda c: c["layers"][0]["mixer"].pop("scale"),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=26),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7),
    lambda c: c["layers"][0]["mixer"]["rot"].update(scaling={"factor": 0.0}),
    lambda c: c["layers"][0]["mixer"]["rot"].update(scaling={"factor": 2.0, "low": 1.0, "high": 4.0, "original": 64}),
    lambda c: c["layers"][0]["mlp"].update(ff=0),
    lambda c: c["layers"][0]["mlp"].update(kind="gated"),
    lambda c: c["layers"][1]["mixer"].update(kv_rank=0),
    lambda c: c["layers"][1]["mixer"]["rot"].update(dims=10),
    lambda c: c["layers"][1]["mlp"]["router"].update(top=7),
    lambda c: c["layers"][1]["mlp"]["expert"].pop("limit"),
    lambda c: c["layers"][1]["mlp"]["shared"].pop("limit"),
    lambda c: c["norm"].update(eps=0),
    lambda c: c.pop("vocab"),
])
def test_what_the_reader_refuses(bad):
    from llmserve.config.model_config import ConfigError
    from llmserve.models.zotunex import ZotunexConfig

    config = copy.deepcopy(SMALL)
    bad(config)
    with pytest.raises(ConfigError):
        ZotunexConfig.from_dict(config)


def test_the_configuration_goes_to_json_and_back():
    from llmserve.models.zotunex import ZotunexConfig

    for config in (SMALL, SMALL_B, SMALL_C, SMALL_D):
        cfg = ZotunexConfig.from_dict(config)
        assert ZotunexConfig.from_dict(cfg.to_dict()) == cfg


def test_a_factor_divides_every_frequency():
    from llmserve.parts.attention_composed import scaled_frequencies

    rot = {"base": 300.0, "dims": 12, "scaling": {"factor": 5.0}}
    got = scaled_frequencies(300.0, 12, {"factor": 5.0})
    assert got == pytest.approx(pz.frequencies(rot).tolist(), rel=1e-15)
    assert got == pytest.approx([f / 5.0 for f in scaled_frequencies(300.0, 12)], rel=1e-15)
    assert scaled_frequencies(10.0, 0, {"factor": 5.0}) == [] and pz.frequencies({"dims": 0, "base": 1.0}).numel() == 0


# ------------------------------------------------------------------------------ the plain mechanisms
def test_the_two_pairings_of_the_rotation():
    """Lengths stay, scores depend on the distance alone, position 0 turns nothing, and the two layouts are one rotation up to
    the order of dimensions."""
    freq = pz.frequencies({"base": 20.0, "dims": 6})
    x = rnd(1, 1, 10, seed=1).expand(9, 1, 10).contiguous()
    pos = torch.arange(9)
    for turn in (pz.rotate_neighbours, pz.rotate_half):
        y = turn(x, freq, pos)
        assert torch.allclose(y.norm(dim=-1), x.norm(dim=-1)) and torch.equal(y[0], x[0]) and torch.equal(y[..., 6:], x[..., 6:])
        dots = y[:, 0] @ y[:, 0].T
        assert torch.allclose(dots[3, 1], dots[8, 6]) and not torch.allclose(dots[3, 1], dots[3, 0])
    order = [0, 3, 1, 4, 2, 5, 6, 7, 8, 9]  # half layout -> neighbours
    assert torch.allclose(pz.rotate_half(x, freq, pos)[..., order], pz.rotate_neighbours(x[..., order], freq, pos))
    angle = float(freq[1]) * 4
    got = pz.rotate_neighbours(x, freq, pos)[4, 0, 2:4]
    u, v = x[4, 0, 2], x[4, 0, 3]
    assert torch.allclose(got, torch.stack([u * math.cos(angle) - v * math.sin(angle), v * math.cos(angle) + u * math.sin(angle)]))


def test_the_sink_is_one_more_term_without_a_value():
    s = rnd(4, 7, seed=2)
    w = pz.softmax_with_sink(s, torch.tensor(1.3, dtype=F64))
    want = torch.softmax(torch.cat([s, torch.full((4, 1), 1.3, dtype=F64)], dim=1), dim=1)[:, :7]
    assert torch.allclose(w, want)


def test_the_correction_decides_and_the_score_weighs():
    t = {"router": torch.tensor([[2.0], [1.0], [0.0]], dtype=F64), "correction": torch.tensor([0.0, -5.0, 1.0], dtype=F64)}
    idx, w = pz.route(torch.ones(1, 1, dtype=F64), t, "", {"top": 2, "scale": 2.5})
    assert idx.tolist() == [[2, 0]]
    assert w[0].tolist() == pytest.approx([2.5 * 0.5, 2.5 / (1 + math.exp(-2.0))])


def test_values_are_the_keys_before_norm_and_rotation():
    """With one token the attention gives back that token's projected key, times the gate."""
    m = {"heads": 2, "kv_heads": 1, "dim": 4, "scale": 0.5, "rot": {"base": 10.0, "dims": 4}}
    t = {"q": rnd(8, 6, seed=3), "k": rnd(4, 6, seed=4), "g": rnd(2, 6, seed=5), "o": torch.eye(8, dtype=F64), "temp": rnd(2, seed=6),
         "q.norm": rnd(4, seed=7), "k.norm": rnd(4, seed=8)}
    h = rnd(1, 6, seed=9)
    k, gate = h @ t["k"].T, torch.sigmoid(h @ t["g"].T)
    assert torch.allclose(pz.attention(h, t, "", m, 1e-5), torch.cat([k * gate[:, :1], k * gate[:, 1:]], dim=1))


def test_the_latent_mixer_is_attention_over_unfolded_keys():
    """Folding W_uk into the query and W_uv behind the sum, as the engine does, is the same mixer."""
    m = {"heads": 2, "dim": 3, "rot_dim": 4, "vdim": 5, "kv_rank": 6, "scale": 0.7, "rot": {"base": 10.0, "dims": 4}}
    t = {"q": rnd(14, 8, seed=10), "dkv": rnd(10, 8, seed=11), "dkv.norm": rnd(6, seed=12), "uk": rnd(6, 6, seed=13),
         "uv": rnd(10, 6, seed=14), "sink": rnd(2, seed=15), "g": rnd(2, 8, seed=16), "o": torch.eye(10, dtype=F64)}
    T = 7
    h = rnd(T, 8, seed=17)
    want = pz.latent_attention(h, t, "", m, 1e-5)
    freq, pos = pz.frequencies(m["rot"]), torch.arange(T)
    q, kv = (h @ t["q"].T).view(T, 2, 7), h @ t["dkv"].T
    c = pz.rms(kv[:, :6], 1e-5, t["dkv.norm"])
    row = torch.cat([c, pz.rotate_half(kv[:, None, 6:], freq, pos)[:, 0]], dim=1)
    qr = pz.rotate_half(q[..., 3:], freq, pos)
    out = []
    for a in range(2):
        folded = torch.cat([q[:, a, :3] @ t["uk"][3 * a: 3 * a + 3], qr[:, a]], dim=1)
        w = pz.softmax_with_sink((folded @ row.T * 0.7).masked_fill(pz.causal(T), -math.inf), t["sink"][a])
        out.append((w @ c) @ t["uv"][5 * a: 5 * a + 5].T * torch.sigmoid(h @ t["g"][a: a + 1].T))
    assert torch.allclose(torch.cat(out, dim=1), want)
