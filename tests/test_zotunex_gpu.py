"""Zotunex on the GPU against the plain implementation (tests/plain_zotunex.py, float64 on the CPU): each mechanism alone,
then whole models of small made-up sizes in every way of cutting a request into steps, with pages that are freed and used
again, and greedy generation through the entry point.

Which experts a token uses is a discrete choice: the 32-bit engine makes the plain implementation's choices, so every
position is compared there.  Whole models in bfloat16 are held to three times what rounding the operands of matrix products
to bfloat16 alone does to the plain logits."""

import math
import random

import pytest
import torch

import plain_zotunex as pz
import traces
from zotunex_configs import SMALL, SMALL_B, SMALL_C, SMALL_D, attention, config_of, dense, latent, moe

pytestmark = pytest.mark.gpu

DEV = torch.device("cuda:0")
DTYPES = [torch.float32, torch.bfloat16]
F64 = torch.float64


def rnd(*shape, seed=0, scale=1.0):
    return scale * torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


def close(got, ref, dtype, what="", loose=1.0):
    got, ref = got.double().cpu(), ref.double()
    assert got.shape == ref.shape, f"{what}: {tuple(got.shape)} vs {tuple(ref.shape)}"
    assert torch.isfinite(got).all(), f"{what}: not finite"
    scale = max(1e-6, float(ref.abs().max()))
    worst = float((got - ref).abs().max()) / scale
    assert worst <= loose * (2.0 ** -6 if dtype == torch.bfloat16 else 2e-5), f"{what}: off by {worst:.2e} of the largest value"


def dev(x, dtype=torch.float32):
    return x.to(dtype).to(DEV).contiguous()


def ints(values):
    return torch.tensor(list(values), dtype=torch.int32, device=DEV)


def in_portions(total, portions):
    a, i = 0, 0
    while a < total:
        n = min(portions[i % len(portions)], total - a)
        i += 1
        yield a, n
        a += n


def shuffled_pages(t, bs, seed=0, spare=3):
    """(number of pages, table [1, n], slots of positions 0 .. t-1)"""
    n = -(-t // bs)
    order = torch.randperm(n + spare, generator=torch.Generator().manual_seed(seed))[:n].tolist()
    return n + spare, ints(order).view(1, -1), [order[p // bs] * bs + p % bs for p in range(t)]


# ------------------------------------------------------------------------------ attention: queries, keys, values
def attention_case(heads, kv, dk, dims, factor, t, seed, dtype, width=32, scale=5.0):
    rot = {"base": 200.0, "dims": dims}
    if factor:
        rot["scaling"] = {"factor": factor}
    m = {"heads": heads, "kv_heads": kv, "dim": dk, "scale": scale / math.sqrt(dk), "rot": rot}
    h = rnd(t, width, seed=seed)
    w = {"q": rnd(heads * dk, width, seed=seed + 1), "k": rnd(kv * dk, width, seed=seed + 2, scale=0.4),
         "g": rnd(heads, width, seed=seed + 3, scale=0.3), "o": torch.eye(heads * dk, dtype=F64),
         "q.norm": rnd(dk, seed=seed + 4, scale=0.3) + 1, "k.norm": rnd(dk, seed=seed + 5, scale=0.3) + 1,
         "temp": rnd(heads, seed=seed + 6, scale=0.3) + 1}
    if dtype == torch.bfloat16:
        h, w = h.to(dtype).double(), {k: v.to(dtype).double() for k, v in w.items()}
    return m, h, w, torch.cat([h @ w["q"].T, h @ w["k"].T, h @ w["g"].T], dim=1)


def run_attention(proj, m, w, eps, dtype, bs, portions=(1000,), kernel="any", angles=True, splits=1, pad=0):
    """The engine's kernels over shuffled pages that hold NaN until they are written.  `kernel`: "any" (attend_composed),
    "composed" (its matrix-core kernel) or "plain" (the plain attention's kernels with gates)."""
    from llmserve.ops import library as ops

    t, heads, kv, dk = proj.shape[0], m["heads"], m["kv_heads"], m["dim"]
    pages, table, slots = shuffled_pages(t, bs)
    k_pool = torch.full((pages, kv, bs, dk), float("nan"), dtype=dtype, device=DEV)
    v_pool = torch.full((pages, kv, dk, bs), float("nan"), dtype=dtype, device=DEV)
    f = pz.frequencies(m["rot"])
    freq = dev(f) if f.numel() else None
    outs = []
    for a, n in in_portions(t, portions):
        p = dev(torch.cat([proj[a: a + n], torch.zeros(n, pad, dtype=F64)], dim=1))
        pos = ints(range(a, a + n))
        q = torch.empty((n, heads * dk), dtype=dtype, device=DEV)
        ops.norm_store(q, p, q_heads=heads, k_heads=kv, dk=dk, v_heads=kv, dv=dk, q_norm=dev(w["q.norm"]), k_norm=dev(w["k.norm"]),
                       eps=eps, positions=pos, slots=ints(slots[a: a + n]), k_pool=k_pool, v_pool=v_pool, block_size=bs, freq=freq,
                       angles=ops.rotary_angles(pos, freq) if angles and freq is not None else None, pairing="neighbours",
                       norm_first=True, q_scale=dev(w["temp"]), values_from_keys=True)
        gate = p[:, (heads + kv) * dk:]
        out = torch.full((n, heads * dk), float("nan"), dtype=dtype, device=DEV)
        one = dict(block_size=bs, scale=float(m["scale"]))
        if kernel == "any":
            ops.attend_composed(out, q, k_pool, v_pool, table, ints([0] * n), pos, heads=heads, kv_heads=kv, dk=dk, dv=dk,
                                gate=gate, gate_heads=True, **one)
        elif kernel == "composed":
            ops.attend_composed_mfma(out, q, k_pool, v_pool, table, ints([0, n]), ints([a + n]), 0, 1, n, heads=heads, kv_heads=kv,
                                     dk=dk, dv=dk, gate=gate, gate_heads=True, **one)
        else:
            ops.attention_mfma(out, q, k_pool, v_pool, table, ints([0, n]), ints([a + n]), 0, 1, n, 0, n, heads, kv, dk,
                               split_waves=n == 1, num_splits=splits, waves=8 if n == 1 and dk <= 160 else 4, head_gate=gate, **one)
        outs.append(out.cpu())
    return torch.cat(outs), k_pool, v_pool, slots


ATTENTION_CASES = [  # heads, kv_heads, dk, turned dimensions, factor, block size, tokens
    (4, 2, 24, 16, 3.0, 8, 90),
    (3, 3, 8, 8, None, 4, 50),
    (5, 1, 28, 0, None, 16, 130),
    (6, 3, 80, 2, 4.0, 16, 70),
    (1, 1, 10, 10, None, 8, 20),
    (8, 2, 64, 30, 2.0, 16, 600),
    (2, 1, 300, 24, 2.0, 8, 40),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv,dk,dims,factor,bs,t", ATTENTION_CASES)
def test_attention_whose_values_are_the_keys(dtype, heads, kv, dk, dims, factor, bs, t):
    """The norm before the rotation in neighbouring pairs, the number per head on the scores, the gate per head; whole and
    in portions down to one token, with the step's table of angles and without, rows that are 16-byte aligned and not."""
    eps = 1e-5
    m, h, w, proj = attention_case(heads, kv, dk, dims, factor, t, 60, dtype)
    want = pz.attention(h, w, "", m, eps)
    got, k_pool, v_pool, slots = run_attention(proj, m, w, eps, dtype, bs)
    close(got, want, dtype, "whole", loose=3)
    # what lies in the cache: keys normed and turned, values as projected, rounded once
    raw = proj[:, heads * dk: (heads + kv) * dk].view(t, kv, dk)
    freq = pz.frequencies(m["rot"])
    turned = pz.rotate_neighbours(pz.rms(raw, eps, w["k.norm"]), freq, torch.arange(t))
    keys = k_pool.permute(0, 2, 1, 3).reshape(-1, kv, dk)[slots]
    values = v_pool.permute(0, 3, 1, 2).reshape(-1, kv, dk)[slots]
    close(keys, turned, dtype, "keys", loose=0.5 if dtype == torch.bfloat16 else 3)
    close(values, raw, dtype, "values", loose=0.5)
    for kwargs in (dict(portions=(7, 2, 1, 19, 1, 1)), dict(portions=(33, 2), angles=False), dict(portions=(40, 3), pad=3)):
        close(run_attention(proj, m, w, eps, dtype, bs, **kwargs)[0], want, dtype, f"{kwargs}", loose=3)


MATRIX_CORE_CASES = [  # heads, kv_heads, dk, turned dimensions, factor, block size, tokens
    (6, 2, 128, 32, 4.0, 16, 300),
    (8, 1, 64, 32, None, 16, 420),
    (6, 3, 80, 16, 2.0, 8, 150),
    (3, 3, 32, 32, None, 16, 70),
    (20, 1, 48, 6, None, 8, 90),
    (2, 1, 192, 64, 3.0, 16, 200),
]


@pytest.mark.parametrize("heads,kv,dk,dims,factor,bs,t", MATRIX_CORE_CASES)
def test_attention_on_the_matrix_cores(heads, kv, dk, dims, factor, bs, t):
    """The plain attention's kernels with a gate per head (prompts, portions, single tokens, keys shared out to several
    workgroups in both) and the composed attention's."""
    eps, dtype = 1e-5, torch.bfloat16
    m, h, w, proj = attention_case(heads, kv, dk, dims, factor, t, 61, dtype)
    want = pz.attention(h, w, "", m, eps)
    runs = [dict(kernel="plain"), dict(kernel="plain", portions=(7, 2, 1, 19, 1, 1, 64)),
            dict(kernel="plain", portions=(t - 40,) + (1,) * 40), dict(kernel="plain", portions=(t - 40,) + (1,) * 40, splits=3),
            dict(kernel="plain", portions=(t // 2, 9, 2), splits=2)]
    if dk <= 128 and heads // kv <= 16:
        runs += [dict(kernel="composed"), dict(kernel="composed", portions=(7, 2, 1, 19, 1, 1, 64))]
    for kwargs in runs:
        close(run_attention(proj, m, w, eps, dtype, bs, **kwargs)[0], want, dtype, f"{kwargs}", loose=3)


@pytest.mark.parametrize("kernel", ["any", "composed", "plain"])
def test_a_far_key_is_found_and_a_wrong_number_per_head_shows(kernel):
    """Unit-RMS queries and keys: a match scores dk * scale, every other key 0.  The one key that matches takes all the
    weight wherever it lies, and the result is its raw value, which its norm does not touch.  A head whose number on the
    scores is 0 weighs all keys alike."""
    dk, bs, t = 16, 16, 700
    dtype = torch.float32 if kernel == "any" else torch.bfloat16
    m = {"heads": 2, "kv_heads": 1, "dim": dk, "scale": 4.0, "rot": {"dims": 0}}
    w = {"q.norm": torch.ones(dk, dtype=F64), "k.norm": torch.ones(dk, dtype=F64), "temp": torch.tensor([1.0, 0.0], dtype=F64)}
    for far in (0, 1, 15, 16, 31, 32, 333, 698, 699):
        q = torch.zeros(t, 2 * dk, dtype=F64)
        q[:, 0] = q[:, dk] = 1.0
        k = torch.zeros(t, dk, dtype=F64)
        k[:, 1] = 1.0
        k[far] = 0.0
        k[far, 0] = 3.0
        z = torch.tensor([[0.0, 60.0]], dtype=F64).expand(t, 2)  # gates 1/2 and 1
        got = run_attention(torch.cat([q, k, z], dim=1), m, w, 1e-6, dtype, bs, portions=(t - 1, 1), kernel=kernel)[0].double()
        assert float(got[t - 1, 0]) == pytest.approx(1.5, rel=1e-2) and abs(float(got[t - 1, 1])) < 1e-2, f"the key at {far}"
        assert float(got[t - 1, dk]) == pytest.approx(3.0 / t, rel=2e-2), "the head that weighs all keys alike"
        assert float(got[t - 1, dk + 1]) == pytest.approx((t - 1) / t, rel=1e-2)


def test_the_other_order_and_pairing_of_norm_and_rotation():
    """What the same kernels give when the rotation comes first or pairs lie a half apart, sizes taken 4 numbers a lane and
    not, beside each other and beside the plain order."""
    from llmserve.ops import library as ops

    n, heads, kv = 21, 3, 2
    pos = ints([0, 1, 2, 700, 5, 31, 1500] * 3)
    positions = pos.cpu().long()
    for dk, dims in ((32, 16), (64, 64), (20, 8), (10, 6), (12, 12)):
        f = pz.frequencies({"base": 30.0, "dims": dims})
        x = rnd(n, heads + kv, dk, seed=dk)
        qw, kw = rnd(dk, seed=1) + 1, rnd(dk, seed=2) + 1
        weights = torch.stack([qw] * heads + [kw] * kv)
        for pairing, turn in (("half", pz.rotate_half), ("neighbours", pz.rotate_neighbours)):
            for norm_first in (False, True):
                normed = x / torch.sqrt((x * x).mean(-1, keepdim=True) + 1e-3) * weights
                if norm_first:
                    want = turn(normed, f, positions)
                else:
                    y = turn(x, f, positions)
                    want = y / torch.sqrt((y * y).mean(-1, keepdim=True) + 1e-3) * weights
                for angles in (False, True):
                    q = torch.empty((n, heads * dk), dtype=torch.float32, device=DEV)
                    k_pool = torch.full((4, kv, 8, dk), float("nan"), dtype=torch.float32, device=DEV)
                    v_pool = torch.full((4, kv, dk, 8), float("nan"), dtype=torch.float32, device=DEV)
                    slots = torch.randperm(32, generator=torch.Generator().manual_seed(3))[:n].tolist()
                    freq = dev(f)
                    ops.norm_store(q, dev(x.reshape(n, -1)), q_heads=heads, k_heads=kv, dk=dk, v_heads=kv, dv=dk, q_norm=dev(qw),
                                   k_norm=dev(kw), eps=1e-3, positions=pos, slots=ints(slots), k_pool=k_pool, v_pool=v_pool,
                                   block_size=8, freq=freq, angles=ops.rotary_angles(pos, freq) if angles else None,
                                   pairing=pairing, norm_first=norm_first, values_from_keys=True)
                    what = f"{dk} {dims} {pairing} {norm_first} {angles}"
                    close(q.view(n, heads, dk), want[:, :heads], torch.float32, what, loose=20)
                    close(k_pool.permute(0, 2, 1, 3).reshape(32, kv, dk)[slots], want[:, heads:], torch.float32, what, loose=20)
                    close(v_pool.permute(0, 3, 1, 2).reshape(32, kv, dk)[slots], x[:, heads:], torch.float32, what)
                    untouched = [s for s in range(32) if s not in slots]
                    assert torch.isnan(k_pool.permute(0, 2, 1, 3).reshape(32, kv, dk)[untouched]).all()
                    assert torch.isnan(v_pool.permute(0, 3, 1, 2).reshape(32, kv, dk)[untouched]).all()


# ------------------------------------------------------------------------------ latent attention
def latent_weights(width, m, seed):
    H, dn, dr, dv, r = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    return {"q": rnd(H * (dn + dr), width, seed=seed, scale=0.5), "dkv": rnd(r + dr, width, seed=seed + 1, scale=0.5),
            "dkv.norm": rnd(r, seed=seed + 2, scale=0.3) + 1, "uk": rnd(H * dn, r, seed=seed + 3, scale=0.3),
            "uv": rnd(H * dv, r, seed=seed + 4, scale=0.3), "sink": rnd(H, seed=seed + 5, scale=2.0),
            "g": rnd(H, width, seed=seed + 6, scale=0.3), "o": rnd(width, H * dv, seed=seed + 7, scale=0.3)}


class OneRequest:
    """What a mixer part reads of a step and its cache, for one request whose pages are shuffled."""

    def __init__(self, t, bs, row, dtype):
        from types import SimpleNamespace

        self.bs = bs
        pages, self.table, self.slots = shuffled_pages(t, bs, seed=4)
        self.cache = SimpleNamespace(group_id=0, store=True, block_size=bs,
                                     k_pool=torch.full((pages, 1, bs, row), float("nan"), dtype=dtype, device=DEV))

    def step(self, a, n):
        from types import SimpleNamespace

        view = SimpleNamespace(block_tables=self.table, slots=ints(self.slots[a: a + n]))
        return SimpleNamespace(groups={0: view}, shared={}, positions=ints(range(a, a + n)), token_seq=ints([0] * n),
                               state_slots=ints([0]), cu_seqlens=ints([0, n]), context_lens=ints([a + n]), num_seqs=1, max_count=n,
                               max_context=a + n, num_decode=int(n == 1), max_decode_context=a + n, num_tokens=n)


def run_latent(h, t, m, eps, dtype, bs, portions, width):
    from llmserve.parts import model  # noqa: F401  (registers the built-in parts)
    from llmserve.models.zotunex import _latent_spec
    from llmserve.parts.registry import MIXERS, BuildContext

    part = MIXERS.build(_latent_spec(m, width, eps), BuildContext(dtype, DEV))
    assert {k: tuple(v.shape) for k, v in part.param_infos().items()} == {k: tuple(v.shape) for k, v in t.items()}
    part.load({k: dev(v, dtype) for k, v in t.items()})
    request = OneRequest(h.shape[0], bs, m["kv_rank"] + m["rot_dim"], dtype)
    return torch.cat([part.forward(dev(h[a: a + n], dtype), request.step(a, n), request.cache).cpu()
                      for a, n in in_portions(h.shape[0], portions)])


LATENT_CASES = [  # heads, dim, rot_dim, turned, vdim, kv_rank, block size, tokens
    (3, 12, 8, 8, 20, 40, 8, 90),
    (1, 8, 8, 4, 80, 16, 16, 40),
    (5, 10, 6, 6, 4, 12, 4, 60),
    (4, 32, 16, 16, 32, 48, 16, 300),
    (8, 16, 32, 32, 48, 160, 16, 200),
    (2, 4, 0, 0, 8, 16, 8, 33),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dn,dr,dims,dv,r,bs,t", LATENT_CASES)
def test_latent_attention_with_a_sink_and_a_gate_per_head(dtype, heads, dn, dr, dims, dv, r, bs, t):
    m = {"heads": heads, "dim": dn, "rot_dim": dr, "vdim": dv, "kv_rank": r, "scale": 0.3, "rot": {"base": 50.0, "dims": dims}}
    width, eps = 32, 1e-5
    w, h = latent_weights(width, m, 100), rnd(t, width, seed=99)
    if dtype == torch.bfloat16:
        h, w = h.to(dtype).double(), {k: v.to(dtype).double() for k, v in w.items()}
    want = pz.latent_attention(h, w, "", m, eps)
    for portions in ((1000,), (7, 2, 1, 19, 1, 1), (t - 20,) + (1,) * 20):
        close(run_latent(h, w, m, eps, dtype, bs, portions, width), want, dtype, f"portions {portions[:6]}", loose=3)


@pytest.mark.parametrize("matrix_cores", [False, True])
@pytest.mark.parametrize("splits", [1, 3])
def test_the_sink_of_a_head_takes_its_share(matrix_cores, splits):
    """Rows at right angles to the query: every score is 0, and head a's sink holds exp(s_a) parts in t + exp(s_a), the scale
    left out of it.  A sink far above every score takes everything, one far below nothing."""
    from llmserve.ops import library as ops

    if splits > 1 and not matrix_cores:
        pytest.skip("the kernel that takes any size shares no keys out")
    r, dr, bs, heads = 16, 16, 16, 4
    dtype = torch.bfloat16 if matrix_cores else torch.float32
    sinks = torch.tensor([1.5, -2.0, -60.0, 90.0], dtype=F64)
    for t in (1, 2, 17, 100, 700):
        pages, table, slots = shuffled_pages(t, bs)
        rows = torch.zeros(pages * bs, r + dr, dtype=F64)
        rows[slots, 1] = torch.arange(t, dtype=F64) * 0.25 / t + 1.0
        pool = dev(rows.view(pages, 1, bs, r + dr), dtype)
        q = torch.zeros(1, heads, r + dr, dtype=F64)
        q[..., 0] = 1.0
        out = torch.full((1, heads * r), float("nan"), dtype=dtype, device=DEV)
        common = dict(heads=heads, r=r, dr=dr, block_size=bs, window=0, scale=0.01, sink=dev(sinks))
        if matrix_cores:
            ops.attend_latent_mfma(out, dev(q.view(1, -1), dtype), pool, table, ints([0, 1]), ints([t]), n_seqs=1, max_count=1,
                                   splits=splits, **common)
        else:
            ops.attend_latent(out, dev(q.view(1, -1), dtype), pool, table, ints([0]), ints([t - 1]), ints([t]), **common)
        want = rows[slots, 1].sum() / (t + torch.exp(sinks))
        got = out.view(heads, r).double().cpu()
        close(got[:, 1], want, dtype, f"{t} rows", loose=1)
        assert float(got[3, 1]) < 1e-30 and float(got[:, 0].abs().max()) == 0.0


@pytest.mark.parametrize("dn,dr,dims,r", [(12, 8, 8, 40), (16, 12, 4, 20), (10, 6, 6, 12), (8, 16, 16, 32), (4, 0, 0, 8)])
@pytest.mark.parametrize("pairing", ["half", "neighbours"])
def test_queries_and_cache_rows_in_one_launch(dn, dr, dims, r, pairing):
    """latent_split against latent_query and latent_prepare, few tokens and many, with the table of angles and without:
    the same bits."""
    from llmserve.ops import library as ops

    heads = 3
    dq = dn + dr
    for n in (5, 1100):
        z = dev(rnd(n, heads * dq + r + dr + heads, seed=5))
        pos = ints(torch.randint(0, 3000, (n,), generator=torch.Generator().manual_seed(6)).tolist())
        slots = ints(torch.randperm(n + 9, generator=torch.Generator().manual_seed(7))[:n].tolist())
        freq = dev(pz.frequencies({"base": 50.0, "dims": dims})) if dims else None
        wc = dev(rnd(r, seed=8) + 1)
        results = []
        for angles in (None, ops.rotary_angles(pos, freq) if dims else None):
            turn = dict(freq=freq, positions=pos, pairing=pairing, angles=angles)
            for split in (True, False):
                plain = torch.empty((n, heads * dn), dtype=torch.bfloat16, device=DEV)
                folded = torch.zeros((n, heads * (r + dr)), dtype=torch.bfloat16, device=DEV)
                pool = torch.zeros((n + 9, 1, 1, r + dr), dtype=torch.bfloat16, device=DEV)
                if split:
                    ops.latent_split(plain, folded, z, col_q=0, col_c=heads * dq, heads=heads, dn=dn, dr=dr, r=r, wc=wc, eps=1e-5,
                                     pool=pool, slots=slots, **turn)
                else:
                    ops.latent_query(plain, folded, z[:, : heads * dq].contiguous(), heads=heads, dn=dn, dr=dr, r=r, **turn)
                    cq = torch.empty((n, 1), dtype=torch.bfloat16, device=DEV)
                    ops.latent_prepare(z, col_q=0, q_rank=1, col_c=heads * dq, r=r, dr=dr, wq=dev(torch.ones(1)), wc=wc, eps=1e-5,
                                       cq=cq, pool=pool, slots=slots, **turn)
                results.append((plain, folded, pool))
        for other in results[1:]:
            assert all(torch.equal(a, b) for a, b in zip(results[0], other))
        q = z[:, : heads * dq].double().cpu().view(n, heads, dq)
        close(results[0][0].view(n, heads, dn), q[..., :dn], torch.bfloat16, "unrotated parts", loose=0.5)
        if dims:
            turn = pz.rotate_half if pairing == "half" else pz.rotate_neighbours
            want = turn(q[..., dn:], pz.frequencies({"base": 50.0, "dims": dims}), pos.cpu())
            close(results[0][1].view(n, heads, r + dr)[..., r:], want, torch.bfloat16, "rotated parts", loose=0.5)


# ------------------------------------------------------------------------------ norms and feed-forwards
@pytest.mark.parametrize("dtype", DTYPES)
def test_a_norm_with_one_number_for_all_coordinates(dtype):
    from llmserve.parts import model  # noqa: F401
    from llmserve.parts.registry import NORMS, BuildContext
    from llmserve.parts.spec import PartSpec

    for width in (44, 72, 512):
        part = NORMS.build(PartSpec("rmsnorm_streams", {"hidden": width, "eps": 1e-3, "tensor": "", "scalar": True}), BuildContext(dtype, DEV))
        assert tuple(part.param_infos()[""].shape) == ()
        part.load({"": torch.tensor(1.75, dtype=dtype, device=DEV)})
        x = rnd(9, width, seed=width, scale=0.05)
        close(part.forward(dev(x)), pz.rms(x, 1e-3, 1.75), dtype, f"width {width}", loose=0.5)


def unit_weights(width, ff, seed, gate=True):
    t = {"up": rnd(ff, width, seed=seed, scale=0.4), "down": rnd(width, ff, seed=seed + 1, scale=0.4)}
    if gate:
        t["gate"] = rnd(ff, width, seed=seed + 2, scale=0.4)
    return t


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,ff", [(64, 96), (44, 30), (128, 512)])
def test_dense_feed_forwards_at_every_row_count(dtype, width, ff):
    """The squared relu between two matrices and the clamped gated unit, through every product the row count chooses; limits
    that cut off most of the units and limits that cut off none."""
    from llmserve.parts import model  # noqa: F401
    from llmserve.parts.registry import FEED_FORWARDS, BuildContext
    from llmserve.parts.spec import PartSpec

    ctx = BuildContext(dtype, DEV)
    t, plain = unit_weights(width, ff, 30), unit_weights(width, ff, 40, gate=False)
    h = rnd(200, width, seed=31)
    if dtype == torch.bfloat16:
        h = h.to(dtype).double()
        t, plain = ({k: v.to(dtype).double() for k, v in x.items()} for x in (t, plain))
    relu = FEED_FORWARDS.build(PartSpec("ungated", {"hidden": width, "intermediate": ff, "activation": "squared_relu",
                                                    "result": "float32"}), ctx)
    assert set(relu.param_infos()) == set(plain)
    relu.load({k: dev(v, dtype) for k, v in plain.items()})
    for rows in (1, 8, 16, 17, 40, 64, 65, 200):
        close(relu.forward(dev(h[:rows], dtype)), pz.squared_relu_unit(h[:rows], plain, ""), dtype, f"squared relu, {rows} rows", loose=2)
    for limit in (0.3, 2.0, 50.0):
        unit = FEED_FORWARDS.build(PartSpec("swiglu", {
            "hidden": width, "intermediate": ff, "result": "float32", "unit": "clamped", "limit": limit,
            "names": {k: k for k in ("gate", "up", "down")}}), ctx)
        unit.load({k: dev(v, dtype) for k, v in t.items()})
        for rows in (1, 8, 16, 17, 40, 64, 65, 200):
            close(unit.forward(dev(h[:rows], dtype)), pz.clamped_unit(h[:rows], t, "", limit), dtype, f"clamped, {rows} rows", loose=2)


@pytest.mark.parametrize("experts,top", [(6, 2), (16, 4), (5, 1), (4, 4), (9, 3)])
def test_the_router_chooses_by_the_corrected_score_and_weighs_by_the_score(experts, top):
    from llmserve.ops import library as ops

    n, width = 60, 24
    h, router = rnd(n, width, seed=80), rnd(experts, width, seed=81, scale=0.3)
    correction = rnd(experts, seed=82, scale=0.4) - 0.6  # corrected scores of either sign
    t = {"router": router, "correction": correction}
    chosen = torch.empty((n, top), dtype=torch.int32, device=DEV)
    weight = torch.empty((n, top), dtype=torch.float32, device=DEV)
    ops.moe_router(chosen, weight, dev(h), dev(router), correction=dev(correction), scale=2.5)
    idx, w = pz.route(h, t, "", {"top": top, "scale": 2.5})
    assert torch.equal(chosen.cpu().long(), idx)
    close(weight, w, torch.float32, "weights", loose=3)
    if top < experts:  # the correction decides: without it other experts are chosen somewhere
        ops.moe_router(chosen, weight, dev(h), dev(router), scale=2.5)
        assert not torch.equal(chosen.cpu().long().sort(dim=1).values, idx.sort(dim=1).values)
    # a correction far below every score, as after long balancing: still the best of what there is
    ops.moe_router(chosen, weight, dev(h), dev(router), correction=dev(correction - 50.0), scale=2.5)
    assert torch.equal(chosen.cpu().long(), pz.route(h, {"router": router, "correction": correction - 50.0}, "", {"top": top, "scale": 1.0})[0])
    # within groups, the corrected scores again
    if experts % 3 == 0:
        keep, per = 1, experts // 3
        few = min(top, per)
        c2, w2 = (torch.empty((n, few), dtype=d, device=DEV) for d in (torch.int32, torch.float32))
        ops.moe_router(c2, w2, dev(h), dev(router), correction=dev(correction), groups=3, keep=keep)
        s = torch.sigmoid(h @ router.T)
        best = (s + correction).view(n, 3, per).max(-1).values.argmax(-1)
        masked = torch.where(torch.arange(experts)[None, :] // per == best[:, None], s + correction, torch.tensor(-math.inf, dtype=F64))
        i2 = masked.topk(few, dim=-1).indices
        assert torch.equal(c2.cpu().long(), i2)
        close(w2, torch.gather(s, 1, i2), torch.float32, "weights within groups", loose=3)


def mixture_weights(width, experts, ff, shared, seed):
    t = {"router": rnd(experts, width, seed=seed), "correction": rnd(experts, seed=seed + 1, scale=0.3)}
    for e in range(experts):
        t.update({f"e{e}.{k}": v for k, v in unit_weights(width, ff, seed + 10 + 3 * e).items()})
    if shared:
        t.update({f"shared.{k}": v for k, v in unit_weights(width, shared, seed + 2).items()})
    return t


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts,top,ff,shared,rows", [(6, 2, 24, 40, 150), (3, 1, 40, 0, 1), (8, 8, 4, 12, 37), (16, 4, 16, 16, 600)])
def test_experts_and_the_shared_expert_against_the_plain_sum(dtype, experts, top, ff, shared, rows):
    from llmserve.models.zotunex import _mlp_spec
    from llmserve.parts import model  # noqa: F401
    from llmserve.parts.registry import FEED_FORWARDS, BuildContext

    width = 32
    mlp = moe(experts, top, ff, limit=0.9, scale=1.8, shared=shared, shared_limit=0.4)
    t, h = mixture_weights(width, experts, ff, shared, 90), rnd(rows, width, seed=91)
    if dtype == torch.bfloat16:
        h, t = h.to(dtype).double(), {k: v.to(dtype).double() for k, v in t.items()}
    part = FEED_FORWARDS.build(_mlp_spec(width, mlp), BuildContext(dtype, DEV))
    assert set(part.param_infos()) == set(t)
    part.load({k: dev(v, dtype) for k, v in t.items()})
    close(part.forward(dev(h, dtype)), pz.mixture(h, t, "", mlp), dtype, "experts", loose=4)


# ------------------------------------------------------------------------------ whole models
def write_model(folder, config, seed):
    from safetensors.torch import load_file, save_file

    from llmserve.weights import write_random_model

    # stored in bfloat16, so that both engines and the plain implementation hold the same numbers
    write_random_model(folder, config, seed=seed, dtype=torch.bfloat16, std=0.12, norm_std=0.05)
    tensors = load_file(str(folder / "model.safetensors"))
    g = torch.Generator().manual_seed(seed)
    for name in tensors:
        if name.endswith(".mlp.router"):  # routers that decide: with logits close together choices are a coin's toss in bfloat16
            tensors[name] = (tensors[name].float() * 8.0).to(torch.bfloat16)
        if name.endswith(".sink"):  # sinks that matter, of either sign
            tensors[name] = (2.0 * torch.randn(tensors[name].shape, generator=g)).to(torch.bfloat16)
        if name.endswith(".temp"):
            tensors[name] = (1.0 + 0.5 * torch.randn(tensors[name].shape, generator=g)).to(torch.bfloat16)
        if name.endswith("norm1") or name.endswith("norm2") or name == "final.norm":
            tensors[name] = (tensors[name].float() * 1.5).to(torch.bfloat16)
    save_file(tensors, str(folder / "model.safetensors"))
    return {k: v.double() for k, v in tensors.items()}


def position_errors(got, ref, scale):
    d = got.double() - ref.double()
    d = d - d.mean(dim=-1, keepdim=True)
    return d.pow(2).mean(dim=-1).sqrt() / scale


def bf16(h):
    return h.to(torch.bfloat16).double()


def logits_close(got, ref, dtype, what, noise=None):
    """Per position: the difference of the logits (mean taken off, root mean square over the vocabulary) against the
    root mean square of the logits themselves.  32-bit: every position.  bfloat16: against `noise`, the plain logits
    with nothing but operands of matrix products rounded to bfloat16, which no bfloat16 engine avoids: the median and the
    upper quartile of the engine's differences stay within three times those of that rounding alone."""
    got, ref = (torch.cat(list(x)) if isinstance(x, (list, tuple)) else x for x in (got, ref))
    scale = ref.double().pow(2).mean().sqrt()
    assert got.shape == ref.shape and torch.isfinite(got).all(), what
    err = position_errors(got, ref, scale)
    worst = int(err.argmax())
    if dtype == torch.float32:
        assert float(err.max()) <= 5e-5, f"{what}: position {worst} is off by {float(err.max()):.2e}"
        return
    floor = position_errors(torch.cat(list(noise)) if isinstance(noise, (list, tuple)) else noise, ref, scale)
    for q in (0.5, 0.75):
        a, b = float(err.quantile(q)), float(floor.quantile(q))
        assert a <= 3.0 * b + 2e-3, f"{what}: quantile {q} of the positions is off by {a:.2e}, rounding alone by {b:.2e}"


MODELS = {"small": (SMALL, 8), "small_b": (SMALL_B, 16), "small_c": (SMALL_C, 4), "small_d": (SMALL_D, 16)}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for i, (name, (config, bs)) in enumerate(MODELS.items()):
        folder = tmp_path_factory.mktemp(f"zotunex_{name}")
        out[name] = (folder, config, write_model(folder, config, seed=170 + i), bs)
    return out


def poison(runner):
    """Pages hold NaN until the engine writes them."""
    runner.storage.poison()


def run_trace(runner, steps):
    from llmserve.engine.replay import Replayer

    rep, outputs = Replayer(runner), {}
    for rec in steps:
        out = rep.run(rec)
        runner.manager.check_invariants()
        if out.shape[0]:
            outputs[rec["step"]] = out.float().cpu()
    return traces.collect(steps, outputs)


def runner_of(folder, **kwargs):
    from llmserve.config import EngineConfig
    from llmserve.engine.runner import ModelRunner

    return ModelRunner.from_folder(folder, EngineConfig(**kwargs))


@pytest.mark.parametrize("name", list(MODELS))
def test_the_stream_after_every_layer(models, name):
    from llmserve.engine.batch import build_batch

    folder, config, w, bs = models[name]
    ids = traces.random_ids(config["vocab"], 45, 5)
    want = []
    pz.forward(config, w, ids, collect=want)
    runner = runner_of(folder, dtype="float32", block_size=bs, num_blocks=16, max_num_seqs=2, use_graphs=False)
    runner.add_sequence("a")
    batch = build_batch(runner.manager.append(["a"], [len(ids)]), [ids], [0], runner._uploader, runner.storage)
    model = runner.model
    x, delta = model.embedding.forward(batch.token_ids), None
    for pos, index in enumerate(model.spec.schedule):
        x, delta = model.blocks[index].forward(x, delta, batch, runner.storage.layer_cache(pos, None))
        close(x[:, 0] + delta.y, want[pos], torch.float32, f"after layer {pos}")


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(MODELS))
@pytest.mark.parametrize("graphs", [True, False])
def test_every_way_of_cutting_gives_the_plain_logits(models, name, dtype_name, graphs):
    folder, config, w, bs = models[name]
    dtype = getattr(torch, dtype_name)
    seqs = {f"r{i}": traces.random_ids(config["vocab"], n, 300 + i) for i, n in enumerate([67, 1, 30, 41, 2, 75])}
    ref = {rid: pz.forward(config, w, ids) for rid, ids in seqs.items()}
    noise = [pz.forward(config, w, ids, rounded=bf16) for ids in seqs.values()] if dtype == torch.bfloat16 else None
    modes = {"whole": traces.whole(seqs), "decode": traces.prefill_then_decode(seqs, tail=40),
             "portions": traces.portions(seqs), "mixed": traces.mixed(seqs, seed=3, live_max=3)}
    for mode, steps in modes.items():
        pages = -(-traces.tokens_needed(steps, round_to=bs) // bs)
        runner = runner_of(folder, dtype=dtype_name, block_size=bs, num_blocks=pages, max_num_seqs=3, use_graphs=graphs)
        assert runner._use_graphs == graphs  # every part of the model can be captured
        poison(runner)
        got = run_trace(runner, steps)
        logits_close([got[rid] for rid in seqs], [ref[rid] for rid in seqs], dtype, f"{name} {mode} {dtype_name}", noise)
        assert runner.manager.num_free_slots == 3
        assert all(a.num_free == pages for a in runner.manager.allocators.values())
        if graphs and mode == "decode":
            assert runner._graphs, "steps of single tokens were not replayed from a graph"


def test_a_batch_gives_each_request_what_it_gets_alone(models):
    folder, config, _w, bs = models["small"]
    seqs = {f"b{i}": traces.random_ids(config["vocab"], n, 500 + i) for i, n in enumerate([50, 13, 29])}
    runner = runner_of(folder, dtype="float32", block_size=bs, num_blocks=64, max_num_seqs=3)
    alone = run_trace(runner, traces.portions(seqs))
    together = run_trace(runner, traces.mixed(seqs, seed=9, live_max=3))
    for rid in seqs:
        assert (alone[rid] - together[rid]).abs().max() <= 2e-5 * float(alone[rid].abs().max())


def test_long_decoding_and_the_prompt_of_the_same_tokens_agree(models):
    """280 tokens: whole in one step, and most of them one by one through the pages; then again on the pages that came
    back."""
    folder, config, w, bs = models["small_c"]
    ids = traces.random_ids(config["vocab"], 280, 77)
    ref = pz.forward(config, w, ids)
    for graphs in (True, False):
        runner = runner_of(folder, dtype="float32", block_size=bs, num_blocks=-(-280 // bs) + 1, max_num_seqs=2, use_graphs=graphs)
        poison(runner)
        got = run_trace(runner, traces.prefill_then_decode({"long": ids}, tail=250))
        logits_close(got["long"], ref, torch.float32, "long decoding")
        whole = run_trace(runner, traces.whole({"again": ids}))
        logits_close(whole["again"], ref, torch.float32, "the whole prompt on the pages that came back")


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
def test_a_long_request_at_matrix_core_sizes(models, dtype_name):
    """650 tokens at sizes the matrix-core kernels take: the prompt in one step and its last tokens one by one (keys shared
    out to several workgroups, several tiles a wave), then in portions on the pages that came back."""
    folder, config, w, bs = models["small_d"]
    dtype = getattr(torch, dtype_name)
    ids = traces.random_ids(config["vocab"], 650, 78)
    ref = pz.forward(config, w, ids)
    noise = pz.forward(config, w, ids, rounded=bf16) if dtype == torch.bfloat16 else None
    runner = runner_of(folder, dtype=dtype_name, block_size=bs, num_blocks=-(-650 // bs) + 1, max_num_seqs=2)
    poison(runner)
    got = run_trace(runner, traces.prefill_then_decode({"long": ids}, tail=48))
    logits_close(got["long"], ref, dtype, f"a long prompt, then token by token, {dtype_name}", noise)
    again = run_trace(runner, traces.portions({"again": ids}, sizes=[200, 7, 2, 130, 64, 1, 33]))
    logits_close(again["again"], ref, dtype, f"the same in portions, {dtype_name}", noise)


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
def test_greedy_generation_through_the_entry_point(models, dtype_name):
    from llmserve import LLM, EngineConfig, SamplingParams

    folder, config, w, bs = models["small"]
    prompts = [traces.random_ids(config["vocab"], n, 600 + i) for i, n in enumerate([19, 3, 33, 8, 1])]
    llm = LLM(folder, dtype=dtype_name, engine=EngineConfig(block_size=bs, num_blocks=40, max_num_seqs=3,
                                                            max_num_batched_tokens=16))
    assert llm.runner.takes_device_tokens  # decode steps are replayed graphs, fed from the sampler's ids
    results = llm.generate(prompts, SamplingParams(max_new_tokens=24))
    for prompt, result in zip(prompts, results):
        assert len(result.tokens) == 24
        ref = pz.forward(config, w, prompt + result.tokens)
        far = 0
        for i, tok in enumerate(result.tokens):
            row = ref[len(prompt) - 1 + i]
            if dtype_name == "float32":  # the plain implementation's own choice, but for a tie within rounding
                far += float(row.max() - row[tok]) > 1e-4 * float(ref.pow(2).mean().sqrt())
            else:
                far += float(row.max() - row[tok]) > 0.25 * float(ref.pow(2).mean().sqrt()) + 1e-3
        assert far <= (0 if dtype_name == "float32" else 2)
    assert llm.runner.manager.num_free_slots == 3


def test_named_sizes_run_from_the_command_line_entry(capsys):
    from llmserve.cli import main

    assert main(["--model", "zotunex-tiny", "--random-weights", "--max-new-tokens", "5", "--dtype", "float32"]) == 0
    assert "decode=" in capsys.readouterr().out


def drawn_config(seed: int) -> tuple[dict, int]:
    """A configuration drawn at random from what config.json allows: the two mixers in any order, both feed-forwards or none,
    with and without a shared expert, 1 to 6 heads, 1 to all of them key/value heads, sizes from 2 up and beyond 64, rotations
    over all, a part or nothing of a head with a factor or without; and a page size."""
    rng = random.Random(seed)

    def rot(within):
        dims = rng.choice([within, within // 2 // 2 * 2, 2, 0])
        r = {"base": rng.choice([10.0, 10000.0, 1e6]), "dims": min(dims, within // 2 * 2)}
        if rng.random() < 0.5 and r["dims"]:
            r["scaling"] = {"factor": rng.choice([2.0, 8.0])}
        return r

    def mlp():
        kind = rng.random()
        if kind < 0.2:
            return None
        if kind < 0.5:
            return dense(rng.choice([8, 30, 96]))
        experts = rng.randint(1, 9)
        return moe(experts, rng.randint(1, min(4, experts)), rng.choice([8, 24, 40]), rng.choice([0.3, 1.0, 7.0]),
                   rng.choice([0.5, 1.0, 2.0]), rng.choice([0, 8, 40]), rng.choice([0.3, 1.5]))

    layers = []
    for _ in range(rng.randint(2, 5)):
        if rng.random() < 0.5:
            dr = rng.choice([2, 4, 8, 16])
            layers.append(latent(mlp(), heads=rng.randint(1, 5), dim=rng.choice([4, 8, 16, 20, 32]), rot_dim=dr,
                                 vdim=rng.choice([4, 8, 16, 40]), kv_rank=rng.choice([8, 16, 32, 48]), scale=rng.choice([0.1, 0.2, 0.35]),
                                 rot=rot(dr)))
        else:
            kv = rng.choice([1, 2, 3])
            dim = rng.choice([4, 10, 16, 32, 48, 64, 96])
            layers.append(attention(mlp(), heads=kv * rng.choice([1, 2, 3]), kv_heads=kv, dim=dim,
                                    scale=rng.choice([0.3, 1.0, 3.0]) / math.sqrt(dim), rot=rot(dim)))
    return config_of(layers, width=rng.choice([40, 64, 72, 100]), vocab=rng.choice([61, 128, 257]), eps=rng.choice([1e-6, 1e-5]),
                     embedding=rng.choice([1.0, 4.0, 12.5])), rng.choice([4, 8, 16])


@pytest.mark.parametrize("seed", list(range(10)))
def test_configurations_drawn_at_random(tmp_path, seed):
    config, bs = drawn_config(seed)
    w = write_model(tmp_path, config, seed=900 + seed)
    seqs = {f"q{i}": traces.random_ids(config["vocab"], n, 40 * seed + i) for i, n in enumerate([90, 3, 47, 160, 18])}
    ref = {rid: pz.forward(config, w, ids) for rid, ids in seqs.items()}
    noise = [pz.forward(config, w, ids, rounded=bf16) for ids in seqs.values()]
    for dtype_name in ("float32", "bfloat16"):
        steps = traces.mixed(seqs, seed=seed, live_max=3, tail=30)
        pages = -(-traces.tokens_needed(steps, round_to=bs) // bs)
        runner = runner_of(tmp_path, dtype=dtype_name, block_size=bs, num_blocks=pages, max_num_seqs=3)
        poison(runner)
        got = run_trace(runner, steps)
        logits_close([got[rid] for rid in seqs], [ref[rid] for rid in seqs], getattr(torch, dtype_name),
                     f"seed {seed} {dtype_name}: {config['layers']}", noise)
        assert runner.manager.num_free_slots == 3
        assert all(a.num_free == pages for a in runner.manager.allocators.values())
