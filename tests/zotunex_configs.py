"""Small Zotunex configurations for the tests: sizes differ from layer to layer, and what a configuration may happen to
make equal or 1 (one head, as many key/value heads as query heads, a rotation over all, a part or nothing of a head, a
factor on the frequencies or none, one expert chosen, every expert chosen, no shared expert, no feed-forward, a latent as
wide as a head) appears both ways."""

from __future__ import annotations

import copy

ATTENTION = {"heads": 4, "kv_heads": 2, "dim": 24, "vdim": 24, "scale": 0.31,
             "rot": {"base": 50.0, "dims": 16, "scaling": {"factor": 3.0}}}
LATENT = {"heads": 3, "dim": 12, "rot_dim": 8, "vdim": 20, "kv_rank": 40, "scale": 0.21, "rot": {"base": 100.0, "dims": 8}}


def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=24, limit=0.8, scale=1.7, shared=40, shared_limit=1.1):
    d = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top, "scale": scale}}
    if shared:
        d["shared"] = {"ff": shared, "limit": shared_limit}
    return d


def _mlp(mlp):
    return moe() if mlp == "default" else mlp


def attention(mlp="default", **changes):
    m = dict(copy.deepcopy(ATTENTION), **changes)
    m["vdim"] = m["dim"]
    return {"type": "attention", "mixer": m, "mlp": _mlp(mlp)}


def latent(mlp="default", **changes):
    return {"type": "latent_attention", "mixer": dict(copy.deepcopy(LATENT), **changes), "mlp": _mlp(mlp)}


def config_of(layers, width=72, vocab=151, eps=1e-5, embedding=3.0) -> dict:
    return {"architecture": "Zotunex", "vocab": vocab, "width": width, "embedding": {"scale": embedding}, "norm": {"eps": eps},
            "layers": layers}


def _small():
    return config_of([attention(dense()), latent(), attention(), latent(dense(40), heads=5, rot_dim=4, rot={"base": 1e4, "dims": 4})])


def _small_b():
    # as many key/value heads as query heads, no factor, all of a head turned; one head; every expert chosen; no shared
    # expert; layers without feed-forward
    layers = [latent(None, heads=1, dim=8, rot_dim=8, vdim=80, kv_rank=16, rot={"base": 10.0, "dims": 8}),
              attention(moe(4, 4, 12, 0.5, 1.0, 0), heads=3, kv_heads=3, dim=8, scale=1.2, rot={"base": 1e4, "dims": 8}),
              attention(None, heads=1, kv_heads=1, dim=20, rot={"base": 100.0, "dims": 2}),
              attention(moe(3, 1, 8, 2.0, 2.5, 8, 0.3), heads=6, kv_heads=2, dim=12, rot={"base": 100.0, "dims": 0})]
    return config_of(layers, width=64, vocab=97, eps=1e-6, embedding=1.0)


def _small_c():
    # one key/value head for all; a part of the rotated part turned, with a factor; a width that is no multiple of 8
    layers = [attention(moe(8, 3, 20, 1.0, 0.6, 12, 2.0), heads=5, kv_heads=1, dim=28, rot={"base": 1e5, "dims": 12, "scaling": {"factor": 8.0}}),
              latent(dense(30), heads=4, dim=8, rot_dim=12, vdim=8, kv_rank=12, rot={"base": 1e6, "dims": 4, "scaling": {"factor": 2.0}}),
              latent(moe(5, 2, 16, 0.7, 3.0, 24, 0.7), heads=2, dim=40, rot_dim=6, vdim=4, kv_rank=24, rot={"base": 30.0, "dims": 6})]
    return config_of(layers, width=44, vocab=131, embedding=7.5)


def _small_d():
    # sizes that the matrix cores take (multiples of 16), pages of 16 keys
    layers = [attention(dense(96), heads=4, kv_heads=2, dim=32, scale=0.2, rot={"base": 1000.0, "dims": 16, "scaling": {"factor": 2.0}}),
              latent(moe(4, 2, 32, 0.9, 1.5, 64, 1.4), heads=4, dim=32, rot_dim=16, vdim=32, kv_rank=48, scale=0.15,
                     rot={"base": 1e4, "dims": 16}),
              attention(moe(8, 2, 32, 0.9, 1.5, 32, 0.6), heads=6, kv_heads=2, dim=64, scale=0.15, rot={"base": 1e5, "dims": 64}),
              latent(dense(64), heads=8, dim=16, rot_dim=32, vdim=48, kv_rank=160, scale=0.17, rot={"base": 500.0, "dims": 32}),
              attention(None, heads=2, kv_heads=2, dim=96, scale=0.12, rot={"base": 100.0, "dims": 48})]
    return config_of(layers, width=64, vocab=173, embedding=2.0)


SMALL, SMALL_B, SMALL_C, SMALL_D = _small(), _small_b(), _small_c(), _small_d()
