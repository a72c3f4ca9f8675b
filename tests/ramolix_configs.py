"""Small Ramolix configurations for the tests: sizes differ from layer to layer, and what a configuration may happen to
make equal or 1 (one head, as many key/value heads as query heads, a rotation over all, a part or nothing of a head, stretched
frequencies or plain ones, a window of one key or none, one group, a group per head, one tap, one normed part, parts across
heads, no feed-forward, layers that read another layer's latents) appears both ways."""

from __future__ import annotations

import copy

STRETCH = {"factor": 3.0, "low": 1.0, "high": 5.0, "original": 64}
SPACE = {"heads": 6, "vdim": 12, "state": 20, "groups": 3, "conv": 4, "norm_groups": 3}
ATTENTION = {"heads": 4, "kv_heads": 2, "dim": 24, "vdim": 24, "scale": 0.31, "mask": {"size": 13},
             "rot": {"base": 50.0, "dims": 16, "scaling": STRETCH}}
LATENT = {"heads": 3, "dim": 12, "vdim": 20, "kv_rank": 40, "scale": 0.4}


def _mlp(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def space(ff=56, **changes):
    return {"type": "mamba2", "mixer": dict(copy.deepcopy(SPACE), **changes), "mlp": _mlp(ff)}


def attention(ff=56, **changes):
    m = dict(copy.deepcopy(ATTENTION), **changes)
    m["vdim"] = m["dim"]
    return {"type": "attention", "mixer": m, "mlp": _mlp(ff)}


def latent(ff=56, **changes):
    return {"type": "latent_attention", "mixer": dict(copy.deepcopy(LATENT), **changes), "mlp": _mlp(ff)}


def config_of(layers, width=72, vocab=151, eps=1e-5, embedding=3.0, mult=0.6) -> dict:
    return {"architecture": "Ramolix", "vocab": vocab, "width": width, "embedding": {"scale": embedding}, "norm": {"eps": eps},
            "residual_mult": mult, "layers": layers}


def _small():
    layers = [latent(), space(), attention(), latent(40, heads=5, dim=8, vdim=8, kv_from=0), space(None, groups=1, norm_groups=1),
              latent(heads=2, dim=16, vdim=6, kv_from=0, scale=0.9)]
    return config_of(layers)


def _small_b():
    # one head; as many key/value heads as query heads; all of a head turned, plain frequencies; a window of one key and none;
    # one tap; a group per head; normed parts that cross heads; no feed-forward
    layers = [attention(None, heads=3, kv_heads=3, dim=8, scale=1.2, rot={"base": 1e4, "dims": 8}, mask={"size": 1}),
              space(30, heads=4, vdim=7, state=3, groups=4, conv=1, norm_groups=2),
              attention(24, heads=1, kv_heads=1, dim=20, rot={"base": 100.0, "dims": 2}, mask=None),
              latent(None, heads=1, dim=8, vdim=80, kv_rank=16),
              space(40, heads=1, vdim=33, state=9, groups=1, conv=2, norm_groups=3),
              attention(8, heads=6, kv_heads=2, dim=10, rot={"base": 100.0, "dims": 0}, mask={"size": 30})]
    return config_of(layers, width=64, vocab=97, eps=1e-6, embedding=1.0, mult=1.0)


def _small_c():
    # one key/value head for all; a width that is no multiple of 8; a latent that two layers of other sizes read; five taps
    layers = [space(20, heads=2, vdim=40, state=5, groups=2, conv=5, norm_groups=8),
              attention(30, heads=5, kv_heads=1, dim=28, rot={"base": 1e5, "dims": 12, "scaling": dict(STRETCH, factor=8.0)}, mask={"size": 40}),
              latent(16, heads=4, dim=8, vdim=8, kv_rank=12), latent(30, heads=2, dim=40, vdim=4, kv_rank=12, kv_from=2, scale=0.2),
              space(24, heads=9, vdim=4, state=70, groups=3, conv=3, norm_groups=1)]
    return config_of(layers, width=44, vocab=131, embedding=7.5, mult=0.25)


def _small_d():
    # sizes that the matrix cores take (multiples of 16), pages of 16 keys
    layers = [space(96, heads=4, vdim=48, state=32, groups=2, norm_groups=4),
              attention(96, heads=8, kv_heads=2, dim=32, scale=0.2, mask={"size": 70},
                        rot={"base": 1000.0, "dims": 16, "scaling": dict(STRETCH, original=512)}),
              latent(64, heads=4, dim=32, vdim=32, kv_rank=48, scale=0.3),
              space(None, heads=2, vdim=80, state=144, groups=1, conv=3, norm_groups=2),
              latent(64, heads=8, dim=16, vdim=48, kv_rank=48, kv_from=2, scale=0.25),
              attention(64, heads=3, kv_heads=3, dim=64, scale=0.15, rot={"base": 1e5, "dims": 64}, mask={"size": 200}),
              space(32, heads=6, vdim=16, state=16, groups=6, conv=2, norm_groups=1)]
    return config_of(layers, width=64, vocab=173, embedding=2.0, mult=0.4)


SMALL, SMALL_B, SMALL_C, SMALL_D = _small(), _small_b(), _small_c(), _small_d()
