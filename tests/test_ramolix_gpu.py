"""Ramolix on the GPU against the plain implementation (tests/plain_ramolix.py, float64 on the CPU): each mechanism alone,
then whole models of small made-up sizes in every way of cutting a request into steps, with pages and slots that are freed and
used again, and greedy generation through the entry point.  Whole models in bfloat16 are held to three times what rounding the
operands of matrix products to bfloat16 alone does to the plain logits."""

import math
import random
from types import SimpleNamespace

import pytest
import torch

import plain_ramolix as pr
import traces
from ramolix_configs import SMALL, SMALL_B, SMALL_C, SMALL_D, STRETCH, attention, config_of, latent, space

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


def bf16(h):
    return h.to(torch.bfloat16).double()


# ------------------------------------------------------------------------------ the state-space recurrence
class Requests:
    """Several requests' state slots as a mixer sees them: slots that belong to nobody hold NaN, a request's own slot holds
    zeros when it is taken; a padding request of length 0 stands among them."""

    def __init__(self, names, numbers, seed=0):
        order = torch.randperm(len(names) + 2, generator=torch.Generator().manual_seed(seed)).tolist()
        self.state = torch.full((len(names) + 2, numbers), float("nan"), dtype=torch.float32, device=DEV)
        self.slot = {name: order[i] for i, name in enumerate(names)}
        self.nobody = order[-1]
        self.length = {name: 0 for name in names}
        for s in self.slot.values():
            self.state[s] = 0.0

    def step(self, counts, padding=True):
        """`counts`: name -> new tokens, in order; the padding request brings two rows behind them."""
        names = list(counts)
        cu, context, slots = [0], [], []
        for name in names:
            self.length[name] += counts[name]
            cu.append(cu[-1] + counts[name])
            context.append(self.length[name])
            slots.append(self.slot[name])
        if padding:
            cu.append(cu[-1] + 2)
            context.append(0)
            slots.append(self.nobody)
        return SimpleNamespace(cu_seqlens=ints(cu), context_lens=ints(context), state_slots=ints(slots), num_seqs=len(slots),
                               max_count=max(counts.values()))


def space_weights(m, seed, scale=0.5):
    H, P, N, G, taps = (m[k] for k in ("heads", "vdim", "state", "groups", "conv"))
    channels = H * P + 2 * G * N
    return {"conv": rnd(channels, taps, seed=seed, scale=scale), "conv.b": rnd(channels, seed=seed + 1, scale=0.2),
            "dt_bias": rnd(H, seed=seed + 2) - 1.0, "A_log": rnd(H, seed=seed + 3), "D": rnd(H, seed=seed + 4),
            "norm": rnd(H * P, seed=seed + 5, scale=0.3) + 1}


def plain_recurrence(u, w, m, round_conv=None):
    """y [T, H P] of one sequence from its products u = [z | x | B | C | dt]."""
    T, H, P, N, G = u.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner, gn = H * P, G * N
    xbc = pr.silu(pr.causal_conv(u[:, inner:2 * inner + 2 * gn], w["conv"], w["conv.b"]))
    if round_conv is not None:
        xbc = round_conv(xbc)
    dt = pr.softplus(u[:, 2 * inner + 2 * gn:2 * inner + 2 * gn + H] + w["dt_bias"])
    y = pr.state_space(xbc[:, :inner].reshape(T, H, P), xbc[:, inner:inner + gn].reshape(T, G, N), xbc[:, inner + gn:].reshape(T, G, N),
                       dt, -torch.exp(w["A_log"]), w["D"])
    return y.reshape(T, inner)


def run_recurrence(streams, w, m, dtype, kernel, cuts, parts=None, eps=1e-5, seed=0):
    """The engine's kernels over several requests.  `streams`: name -> u [T, columns]; `cuts`: list of {name: tokens} steps.
    Returns name -> (y, gated and normed rows)."""
    from llmserve.ops import library as ops

    H, P, N, G, taps = (m[k] for k in ("heads", "vdim", "state", "groups", "conv"))
    inner, channels = H * P, H * P + 2 * G * N
    numbers = inner * N + (taps - 1) * channels
    requests = Requests(list(streams), numbers + -numbers % 4, seed=seed)
    args = dict(col=inner, dt_col=inner + channels, taps_w=dev(w["conv"]), bias=dev(w["conv.b"]), dt_bias=dev(w["dt_bias"]),
                a_log=dev(w["A_log"]), d_skip=dev(w["D"]), heads=H, groups=G, p=P, n_states=N, state=requests.state, scan_offset=0,
                ring_offset=inner * N)
    at = {name: 0 for name in streams}
    ys, outs = {name: [] for name in streams}, {name: [] for name in streams}
    for counts in cuts:
        batch = requests.step(counts)
        rows = torch.cat([streams[n][at[n]: at[n] + c] for n, c in counts.items()] +
                         [torch.full((2, next(iter(streams.values())).shape[1]), float("nan"), dtype=F64)])
        u = dev(rows)
        y = torch.full((rows.shape[0], inner), float("nan"), dtype=torch.float32, device=DEV)
        if kernel == "runs":
            ops.space_runs(y, u, batch=batch, **args)
        else:
            ops.space_scan(y, u, dtype=dtype, batch=batch, **args)
        out = torch.full((rows.shape[0], inner), float("nan"), dtype=dtype, device=DEV)
        ops.space_finish(out, y, u, dev(w["norm"]), parts=parts or m["norm_groups"], eps=eps, u=u, col=inner, taps=taps,
                         channels=channels, state=requests.state, ring_offset=inner * N, batch=batch)
        row = 0
        for n, c in counts.items():
            ys[n].append(y[row: row + c].cpu())
            outs[n].append(out[row: row + c].cpu())
            at[n] += c
            row += c
    foreign = [s for s in range(requests.state.shape[0]) if s not in requests.slot.values()]
    assert torch.isnan(requests.state[foreign]).all(), "a slot of nobody was written"
    return {n: (torch.cat(ys[n]), torch.cat(outs[n])) for n in streams}


SPACE_CASES = [  # heads, columns, states, groups, taps, normed parts
    (6, 12, 20, 3, 4, 3),
    (4, 7, 3, 4, 1, 2),
    (1, 33, 9, 1, 2, 1),
    (9, 4, 70, 3, 3, 1),
    (2, 40, 5, 2, 5, 8),
    (4, 16, 32, 1, 4, 4),
    (2, 48, 256, 2, 3, 1),
    (3, 30, 130, 1, 9, 5),
]
RUN_CASES = [
    (4, 48, 32, 2, 4, 4),
    (6, 16, 16, 6, 2, 1),
    (2, 80, 144, 1, 3, 2),
    (8, 64, 128, 2, 4, 2),
    (1, 32, 256, 1, 1, 1),
    (2, 144, 48, 1, 8, 3),
]


def space_of(case):
    return dict(zip(("heads", "vdim", "state", "groups", "conv", "norm_groups"), case))


def space_streams(m, lengths, seed):
    columns = 2 * m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"] + m["heads"]
    columns += -columns % 8
    return {name: rnd(t, columns, seed=seed + i) for i, (name, t) in enumerate(lengths.items())}


CUTS = {  # three requests of 45, 20 and 31 tokens
    "together": [{"a": 45, "b": 20, "c": 31}],
    "portions": [{"a": 7}, {"b": 1, "a": 2}, {"c": 3, "a": 20, "b": 4}, {"a": 1, "c": 2}, {"b": 15, "c": 25, "a": 13}, {"a": 1}, {"a": 1, "c": 1}],
    "one by one": [{"a": 30, "b": 5, "c": 16}] + [{"a": 1, "b": 1, "c": 1}] * 15,
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", SPACE_CASES)
def test_the_recurrence_token_by_token(dtype, case):
    m = space_of(case)
    w, streams = space_weights(m, 10), space_streams(m, {"a": 45, "b": 20, "c": 31}, 50)
    inner = m["heads"] * m["vdim"]
    for name, cuts in CUTS.items():
        got = run_recurrence(streams, w, m, dtype, "scan", cuts)
        for r, u in streams.items():
            want = plain_recurrence(u, w, m, None if dtype == torch.float32 else bf16)
            # (bfloat16: x, B and C are rounded once, where a tie may fall either way, and nothing else is)
            close(got[r][0], want, dtype, f"{name} {r}", loose=1 if dtype == torch.float32 else 0.3)
            normed = pr.gated_group_norm(got[r][0].double(), u[:, :inner], w["norm"], m["norm_groups"], 1e-5)
            close(got[r][1], normed, dtype, f"{name} {r}: gate and norm", loose=0.4 if dtype == torch.bfloat16 else 1)


@pytest.mark.parametrize("case", RUN_CASES)
def test_the_recurrence_in_runs_is_the_recurrence_token_by_token(case):
    """Both round x, B and C once and keep everything else in 32-bit, so they agree far closer than bfloat16 numbers do."""
    m = space_of(case)
    w, streams = space_weights(m, 20), space_streams(m, {"a": 45, "b": 20, "c": 31}, 60)
    for name, cuts in CUTS.items():
        runs = run_recurrence(streams, w, m, torch.bfloat16, "runs", cuts)
        scan = run_recurrence(streams, w, m, torch.bfloat16, "scan", cuts, seed=1)
        for r, u in streams.items():
            close(runs[r][0], scan[r][0], torch.float32, f"{name} {r}", loose=1)
            close(runs[r][0], plain_recurrence(u, w, m, bf16), torch.bfloat16, f"{name} {r} against the plain one", loose=0.3)
            close(runs[r][1], scan[r][1].float(), torch.bfloat16, f"{name} {r}: what leaves", loose=0.5)


@pytest.mark.parametrize("total", [17, 126, 127, 128, 129, 130, 255, 256, 257, 400])
def test_runs_of_every_length_and_their_edges(total):
    """Portions that end just before, on and behind a run's last token, started from nothing and from a state, two requests at
    once whose runs lie side by side in the workspace."""
    m = space_of((4, 16, 32, 2, 4, 2))
    w, streams = space_weights(m, 30), space_streams(m, {"a": total, "b": total + 3}, 70 + total)
    scan = run_recurrence(streams, w, m, torch.bfloat16, "scan", [{"a": total, "b": total + 3}])
    first = total // 3
    for cuts in ([{"a": total, "b": total + 3}], [{"b": 2, "a": first}, {"a": total - first, "b": total + 1}]):
        got = run_recurrence(streams, w, m, torch.bfloat16, "runs", cuts)
        for r in streams:
            close(got[r][0], scan[r][0], torch.float32, f"{r} {cuts}", loose=1)


@pytest.mark.parametrize("kernel", ["scan", "runs"])
def test_a_state_that_must_last(kernel):
    """One token writes, 700 tokens later one token reads: decays so slow that the state must be carried, through portions
    of any size; a request whose decay is fast has forgotten."""
    m = {"heads": 2, "vdim": 16, "state": 16, "groups": 1, "conv": 1, "norm_groups": 1}
    channels = 32 + 32
    w = {"conv": torch.ones(channels, 1, dtype=F64), "conv.b": torch.zeros(channels, dtype=F64), "dt_bias": torch.zeros(2, dtype=F64),
         "A_log": torch.tensor([math.log(1e-3), math.log(2.0)], dtype=F64), "D": torch.zeros(2, dtype=F64), "norm": torch.ones(32, dtype=F64)}
    T = 701
    u = torch.zeros(T, 32 + channels + 8, dtype=F64)
    u[0, 32:64] = 30.0      # x
    u[0, 64] = 25.0         # B
    u[-1, 80] = 20.0        # C
    u[:, 96:98] = 0.5       # dt
    want = plain_recurrence(u, w, m, bf16)
    for cuts in ([{"a": T}], [{"a": 300}, {"a": 2}, {"a": 130}, {"a": 17}, {"a": 251}, {"a": 1}], [{"a": 600}] + [{"a": 1}] * 101):
        y = run_recurrence({"a": u}, w, m, torch.bfloat16, kernel, cuts)["a"][0].double()
        assert float(want[-1, 0]) > 100.0 and abs(float(y[-1, 0]) / float(want[-1, 0]) - 1.0) < 1e-4, f"{len(cuts)} steps"
        assert float(y[-1, 16:].abs().max()) < 1e-6 * float(y[-1, 0])


@pytest.mark.parametrize("kernel", ["scan", "runs"])
def test_decays_of_every_strength(kernel):
    """Step sizes from nothing to hundreds in one run: the logarithms add up to tens of thousands, and the difference of two
    such sums must still be right between neighbours that hardly decay."""
    m = space_of((2, 16, 16, 1, 2, 1))
    w = space_weights(m, 40)
    w["A_log"] = torch.tensor([3.0, -6.0], dtype=F64)
    streams = space_streams(m, {"a": 260}, 80)
    u = streams["a"]
    dt = 2 * 32 + 32
    u[:, dt] = torch.where(torch.arange(260) % 7 == 0, 300.0, -12.0)
    u[:, dt + 1] = torch.where(torch.arange(260) % 50 == 0, 400.0, -9.0)
    want = plain_recurrence(u, w, m, bf16)
    y = run_recurrence(streams, w, m, torch.bfloat16, kernel, [{"a": 140}, {"a": 120}])["a"][0]
    err = (y.double() - want).abs() / want.abs().max(dim=0, keepdim=True).values
    assert torch.isfinite(y).all() and float(err.max()) < 2.0 ** -7 and float(err.median()) < 1e-6


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,parts", [(48, 3), (52, 4), (30, 5), (1024, 2), (1536, 1), (4096, 2), (4100, 1), (4608, 3), (2050, 2), (3072, 2)])
def test_gate_and_norm_in_parts(dtype, width, parts):
    from llmserve.ops import library as ops

    n = 11
    y, z, w = rnd(n, width, seed=1, scale=0.3), rnd(n, width + 4, seed=2, scale=2.0), rnd(width, seed=3) + 1
    y[3] = 0.0
    batch = Requests(["a"], 4).step({"a": n}, padding=False)
    out = torch.empty((n, width), dtype=dtype, device=DEV)
    zd = dev(z)
    ops.space_finish(out, dev(y), zd, dev(w), parts=parts, eps=1e-3, u=zd, col=0, taps=1, channels=1,
                     state=torch.zeros(3, 4, device=DEV), ring_offset=0, batch=batch)
    close(out, pr.gated_group_norm(y, z[:, :width], w, parts, 1e-3), dtype, f"{width} in {parts}", loose=0.5)


@pytest.mark.parametrize("taps", [2, 4, 7])
def test_the_ring_holds_the_last_rows_whatever_the_portions(taps):
    """After every step the ring holds the request's last taps - 1 input rows at their positions' places."""
    m = {"heads": 2, "vdim": 4, "state": 4, "groups": 1, "conv": taps, "norm_groups": 1}
    from llmserve.ops import library as ops

    channels, inner = 16, 8
    w = space_weights(m, 5)
    requests = Requests(["a", "b"], inner * 4 + (taps - 1) * channels)
    u = {n: rnd(40, 40, seed=i) for i, n in enumerate("ab")}
    at = {"a": 0, "b": 0}
    for counts in ({"a": 1}, {"a": 2, "b": 9}, {"b": 1, "a": 1}, {"a": 12}, {"b": 3}, {"b": 1, "a": 1}):
        batch = requests.step(counts, padding=False)
        rows = dev(torch.cat([u[n][at[n]: at[n] + c] for n, c in counts.items()]))
        y, out = torch.zeros(rows.shape[0], inner, device=DEV), torch.zeros(rows.shape[0], inner, device=DEV)
        ops.space_finish(out, y, rows, dev(w["norm"]), parts=1, eps=1e-5, u=rows, col=inner, taps=taps, channels=channels,
                         state=requests.state, ring_offset=inner * 4, batch=batch)
        for n, c in counts.items():
            at[n] += c
            ring = requests.state[requests.slot[n], inner * 4:].view(taps - 1, channels).cpu().double()
            for p in range(max(0, at[n] - taps + 1), at[n]):
                assert torch.equal(ring[p % (taps - 1)], u[n][p, inner:inner + channels].float().double()), f"{n} position {p}"


# ------------------------------------------------------------------------------ attention: queries, keys, values, window
def attention_case(heads, kv, dk, dims, stretch, window, t, seed, dtype, width=32, scale=4.0):
    rot = {"base": 200.0, "dims": dims}
    if stretch:
        rot["scaling"] = STRETCH
    m = {"heads": heads, "kv_heads": kv, "dim": dk, "scale": scale / math.sqrt(dk), "rot": rot,
         "mask": {"size": window} if window else None}
    h = rnd(t, width, seed=seed)
    w = {"q": rnd(heads * dk, width, seed=seed + 1), "k": rnd(kv * dk, width, seed=seed + 2, scale=0.4), "q.b": rnd(heads * dk, seed=seed + 3),
         "k.b": rnd(kv * dk, seed=seed + 4), "o": torch.eye(heads * dk, dtype=F64), "q.norm": rnd(heads * dk, seed=seed + 5, scale=0.3) + 1,
         "k.norm": rnd(kv * dk, seed=seed + 6, scale=0.3) + 1}
    if dtype == torch.bfloat16:
        h, w = h.to(dtype).double(), {k: v.to(dtype).double() for k, v in w.items()}
    return m, h, w, torch.cat([h @ w["q"].T, h @ w["k"].T], dim=1)


def run_attention(proj, m, w, eps, dtype, bs, portions=(1000,), kernel="any", angles=True, splits=1, pad=0):
    """The engine's kernels over shuffled pages that hold NaN until they are written.  `kernel`: "any" (attend_composed),
    "composed" (its matrix-core kernel) or "plain" (the plain attention's kernels)."""
    from llmserve.ops import library as ops

    t, heads, kv, dk = proj.shape[0], m["heads"], m["kv_heads"], m["dim"]
    window = int((m.get("mask") or {}).get("size") or 0)
    pages, table, slots = shuffled_pages(t, bs)
    k_pool = torch.full((pages, kv, bs, dk), float("nan"), dtype=dtype, device=DEV)
    v_pool = torch.full((pages, kv, dk, bs), float("nan"), dtype=dtype, device=DEV)
    f = pr.frequencies(m["rot"])
    freq = dev(f) if f.numel() else None
    bias = dev(torch.cat([w["q.b"], w["k.b"]])) if "q.b" in w else None
    outs = []
    for a, n in in_portions(t, portions):
        p = dev(torch.cat([proj[a: a + n], torch.zeros(n, pad, dtype=F64)], dim=1))
        pos = ints(range(a, a + n))
        q = torch.empty((n, heads * dk), dtype=dtype, device=DEV)
        ops.norm_store(q, p, q_heads=heads, k_heads=kv, dk=dk, v_heads=kv, dv=dk, q_norm=dev(w["q.norm"]), k_norm=dev(w["k.norm"]),
                       eps=eps, positions=pos, slots=ints(slots[a: a + n]), k_pool=k_pool, v_pool=v_pool, block_size=bs, freq=freq,
                       angles=ops.rotary_angles(pos, freq) if angles and freq is not None else None, norm_first=True,
                       values_from_keys=True, joint=True, bias=bias)
        out = torch.full((n, heads * dk), float("nan"), dtype=dtype, device=DEV)
        one = dict(block_size=bs, scale=float(m["scale"]))
        if kernel == "any":
            ops.attend_composed(out, q, k_pool, v_pool, table, ints([0] * n), pos, heads=heads, kv_heads=kv, dk=dk, dv=dk,
                                window=window, **one)
        elif kernel == "composed":
            ops.attend_composed_mfma(out, q, k_pool, v_pool, table, ints([0, n]), ints([a + n]), 0, 1, n, heads=heads, kv_heads=kv,
                                     dk=dk, dv=dk, window=window, **one)
        else:
            ops.attention_mfma(out, q, k_pool, v_pool, table, ints([0, n]), ints([a + n]), 0, 1, n, 0, n, heads, kv, dk, window=window,
                               split_waves=n == 1, num_splits=splits, waves=8 if n == 1 and dk <= 160 else 4, **one)
        outs.append(out.cpu())
    return torch.cat(outs), k_pool, v_pool, slots


ATTENTION_CASES = [  # heads, kv_heads, dk, turned dimensions, stretched, window, block size, tokens
    (4, 2, 24, 16, True, 13, 8, 90),
    (3, 3, 8, 8, False, 1, 4, 50),
    (5, 1, 28, 0, False, 40, 16, 130),
    (6, 3, 80, 2, True, None, 16, 70),
    (1, 1, 10, 10, False, 7, 8, 20),
    (8, 2, 64, 32, True, 100, 16, 600),
    (40, 8, 32, 16, False, 33, 16, 60),
    (2, 1, 256, 24, True, 9, 8, 40),
    (3, 1, 128, 128, True, 2, 16, 50),
    (9, 9, 16, 8, False, 21, 8, 64),
    (20, 20, 256, 64, False, 5, 8, 12),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv,dk,dims,stretch,window,bs,t", ATTENTION_CASES)
def test_attention_normed_over_all_heads_whose_values_are_the_keys(dtype, heads, kv, dk, dims, stretch, window, bs, t):
    """Biases, the norm over all heads of q and of k before the rotation, the window; whole and in portions down to one
    token, with the step's table of angles and without, rows that are 16-byte aligned and not."""
    eps = 1e-5
    m, h, w, proj = attention_case(heads, kv, dk, dims, stretch, window, t, 60, dtype)
    want = pr.attention(h, w, "", m, eps)
    got, k_pool, v_pool, slots = run_attention(proj, m, w, eps, dtype, bs)
    close(got, want, dtype, "whole", loose=3)
    # what lies in the cache: keys normed and turned, values as projected (with the bias), rounded once
    raw = proj[:, heads * dk:] + w["k.b"]
    turned = pr.rotate_half(pr.rms(raw, eps, w["k.norm"]).view(t, kv, dk), pr.frequencies(m["rot"]), torch.arange(t))
    keys = k_pool.permute(0, 2, 1, 3).reshape(-1, kv, dk)[slots]
    values = v_pool.permute(0, 3, 1, 2).reshape(-1, kv, dk)[slots]
    close(keys, turned, dtype, "keys", loose=0.5 if dtype == torch.bfloat16 else 3)
    close(values, raw.view(t, kv, dk), dtype, "values", loose=0.5)
    assert int(torch.isnan(k_pool).sum()) == k_pool.numel() - t * kv * dk
    for kwargs in (dict(portions=(7, 2, 1, 19, 1, 1)), dict(portions=(33, 2), angles=False), dict(portions=(40, 3), pad=3)):
        close(run_attention(proj, m, w, eps, dtype, bs, **kwargs)[0], want, dtype, f"{kwargs}", loose=3)


MATRIX_CORE_CASES = [  # heads, kv_heads, dk, turned dimensions, stretched, window, block size, tokens
    (6, 2, 128, 32, True, 90, 16, 300),
    (8, 1, 64, 32, False, None, 16, 420),
    (6, 3, 80, 16, True, 17, 8, 150),
    (3, 3, 32, 32, False, 1, 16, 70),
    (20, 1, 48, 6, False, 64, 8, 90),
    (2, 1, 192, 64, True, 31, 16, 200),
]


@pytest.mark.parametrize("heads,kv,dk,dims,stretch,window,bs,t", MATRIX_CORE_CASES)
def test_attention_on_the_matrix_cores(heads, kv, dk, dims, stretch, window, bs, t):
    """The plain attention's kernels with a window (prompts, portions, single tokens, keys shared out to several workgroups
    in both) and the composed attention's."""
    eps, dtype = 1e-5, torch.bfloat16
    m, h, w, proj = attention_case(heads, kv, dk, dims, stretch, window, t, 61, dtype)
    want = pr.attention(h, w, "", m, eps)
    runs = [dict(kernel="plain"), dict(kernel="plain", portions=(7, 2, 1, 19, 1, 1, 64)),
            dict(kernel="plain", portions=(t - 40,) + (1,) * 40)]
    if window is None:
        runs += [dict(kernel="plain", portions=(t // 2, 9, 2), splits=2), dict(kernel="plain", portions=(t - 40,) + (1,) * 40, splits=3)]
    else:  # (keys of portions behind a window are not shared out; those of single tokens are)
        runs += [dict(kernel="plain", portions=(1,) * 60, splits=3)]
    if dk <= 128 and heads // kv <= 16:
        runs += [dict(kernel="composed"), dict(kernel="composed", portions=(7, 2, 1, 19, 1, 1, 64))]
    for kwargs in runs:
        close(run_attention(proj, m, w, eps, dtype, bs, **kwargs)[0], want, dtype, f"{kwargs}", loose=3)


@pytest.mark.parametrize("kernel", ["any", "composed", "plain"])
@pytest.mark.parametrize("window", [1, 2, 16, 17, 100, 256])
def test_a_key_just_inside_the_window_takes_all_the_weight_and_one_just_outside_none(kernel, window):
    """Queries and keys of root mean square 1 over both heads: a match scores far above everything else.  The one key that
    matches takes all the weight of every query that sees it, in prompts and in decoding, at a page's border too, and the
    result is its raw value; a query one token later gets nothing of it."""
    dk, bs, t = 16, 16, 400
    dtype = torch.float32 if kernel == "any" else torch.bfloat16
    m = {"heads": 2, "kv_heads": 1, "dim": dk, "scale": 6.0, "rot": {"dims": 0}, "mask": {"size": window}}
    w = {"q.norm": torch.ones(2 * dk, dtype=F64), "k.norm": torch.ones(dk, dtype=F64)}
    for far in (0, 1, 15, 16, 33, 112, 127):
        q = torch.zeros(t, 2 * dk, dtype=F64)
        q[:, 0] = q[:, dk] = 1.0
        k = torch.zeros(t, dk, dtype=F64)
        k[:, 1] = 1.0
        k[far] = 0.0
        k[far, 0] = 3.0
        proj = torch.cat([q, k], dim=1)
        last = min(t - 1, far + window - 1)
        for portions in ((t,), (max(1, last - 1), 1, 1, 1, 50), (far + 1, 2, 64, 1)):
            got = run_attention(proj, m, w, 1e-6, dtype, bs, portions=portions, kernel=kernel)[0].double()
            for i in {far, (far + last) // 2, last}:
                assert float(got[i, 0]) == pytest.approx(3.0, rel=1e-2) and abs(float(got[i, 1])) < 1e-2, f"key {far}, query {i}, {portions}"
                assert float(got[i, dk]) == pytest.approx(3.0, rel=1e-2)
            if last + 1 < t:
                assert abs(float(got[last + 1, 0])) < 1e-6 and float(got[last + 1, 1]) == pytest.approx(1.0, rel=1e-2), \
                    f"key {far} seen by {last + 1}, {portions}"


def test_one_norm_over_all_heads_is_not_a_norm_per_head():
    """A head far larger than the others takes the others' share of the norm; heads alike leave each what it was."""
    from llmserve.ops import library as ops

    heads, dk, n = 4, 16, 3
    x = rnd(n, (heads + heads) * dk, seed=4)
    x[1, :dk] *= 50.0
    q = torch.empty((n, heads * dk), dtype=torch.float32, device=DEV)
    ops.norm_store(q, dev(x), q_heads=heads, k_heads=heads, dk=dk, v_heads=heads, dv=dk, eps=1e-5, norm_first=True,
                   values_from_keys=True, joint=True, q_norm=dev(torch.ones(heads * dk)), k_norm=dev(torch.ones(heads * dk)))
    want = pr.rms(x[:, : heads * dk], 1e-5)
    close(q, want, torch.float32)
    assert float(q[1, dk:].abs().max()) < 0.3 < float(q[0, dk:].abs().max())


# ------------------------------------------------------------------------------ latent attention
def latent_weights(width, m, seed, own=True):
    H, d, dv, r = (m[k] for k in ("heads", "dim", "vdim", "kv_rank"))
    w = {"q": rnd(H * d, width, seed=seed, scale=0.5), "uk": rnd(H * d, r, seed=seed + 3, scale=0.3),
         "uv": rnd(H * dv, r, seed=seed + 4, scale=0.3), "o": rnd(width, H * dv, seed=seed + 7, scale=0.3)}
    if own:
        w |= {"dkv": rnd(r, width, seed=seed + 1, scale=0.5), "dkv.norm": rnd(r, seed=seed + 2, scale=0.3) + 1}
    return w


class OneRequest:
    """What a mixer part reads of a step and its cache, for one request whose pages are shuffled."""

    def __init__(self, t, bs, row, dtype):
        pages, self.table, self.slots = shuffled_pages(t, bs, seed=4)
        pool = torch.full((pages, 1, bs, row), float("nan"), dtype=dtype, device=DEV)
        self.cache = SimpleNamespace(group_id=0, store=True, block_size=bs, k_pool=pool)
        self.reader = SimpleNamespace(group_id=0, store=False, block_size=bs, k_pool=pool)

    def step(self, a, n):
        view = SimpleNamespace(block_tables=self.table, slots=ints(self.slots[a: a + n]))
        return SimpleNamespace(groups={0: view}, shared={}, positions=ints(range(a, a + n)), token_seq=ints([0] * n),
                               state_slots=ints([0]), cu_seqlens=ints([0, n]), context_lens=ints([a + n]), num_seqs=1, max_count=n,
                               max_context=a + n, num_decode=int(n == 1), max_decode_context=a + n, num_tokens=n)


def latent_part(m, w, eps, dtype, width):
    from llmserve.models.ramolix import _latent_spec
    from llmserve.parts import model  # noqa: F401  (registers the built-in parts)
    from llmserve.parts.registry import MIXERS, BuildContext

    part = MIXERS.build(_latent_spec(m, width, eps), BuildContext(dtype, DEV))
    assert {k: tuple(v.shape) for k, v in part.param_infos().items()} == {k: tuple(v.shape) for k, v in w.items()}
    part.load({k: dev(v, dtype) for k, v in w.items()})
    return part


LATENT_CASES = [  # heads, dim, vdim of the owner; of the reader; kv_rank, block size, tokens
    ((3, 12, 20), (5, 8, 4), 40, 8, 90),
    ((1, 8, 80), (2, 40, 8), 16, 16, 40),
    ((5, 10, 4), (1, 6, 30), 12, 4, 60),
    ((4, 32, 32), (8, 16, 48), 48, 16, 300),
    ((8, 16, 48), (2, 64, 16), 160, 16, 200),
    ((2, 4, 8), (3, 4, 8), 8, 8, 33),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("own,reads,r,bs,t", LATENT_CASES)
def test_latents_and_a_layer_that_reads_another_layers(dtype, own, reads, r, bs, t):
    """The owner stores its latents, the reader projects the same rows with matrices, heads and sizes of its own."""
    width, eps = 32, 1e-5
    ma = dict(zip(("heads", "dim", "vdim"), own), kv_rank=r, scale=0.4)
    mb = dict(zip(("heads", "dim", "vdim"), reads), kv_rank=r, scale=0.7, kv_from=0)
    wa, wb = latent_weights(width, ma, 100), latent_weights(width, mb, 200, own=False)
    ha, hb = rnd(t, width, seed=98), rnd(t, width, seed=99)
    if dtype == torch.bfloat16:
        ha, hb = bf16(ha), bf16(hb)
        wa, wb = {k: bf16(v) for k, v in wa.items()}, {k: bf16(v) for k, v in wb.items()}
    c = pr.latents(ha, wa, "", eps)
    want_a, want_b = pr.latent_attention(ha, c, wa, "", ma), pr.latent_attention(hb, c, wb, "", mb)
    for portions in ((1000,), (7, 2, 1, 19, 1, 1), (t - 20,) + (1,) * 20):
        a, b = latent_part(ma, wa, eps, dtype, width), latent_part(mb, wb, eps, dtype, width)
        request = OneRequest(t, bs, r, dtype)
        got_a, got_b = [], []
        for at, n in in_portions(t, portions):
            step = request.step(at, n)
            got_a.append(a.forward(dev(ha[at: at + n], dtype), step, request.cache).cpu())
            got_b.append(b.forward(dev(hb[at: at + n], dtype), step, request.reader).cpu())
        close(torch.cat(got_a), want_a, dtype, f"owner, portions {portions[:6]}", loose=3)
        close(torch.cat(got_b), want_b, dtype, f"reader, portions {portions[:6]}", loose=3)


@pytest.mark.parametrize("matrix_cores", [False, True])
@pytest.mark.parametrize("splits", [1, 3])
def test_a_far_latent_is_found(matrix_cores, splits):
    """One row that matches the query takes all the weight wherever it lies: the first, around a page's border, far back."""
    from llmserve.ops import library as ops

    if splits > 1 and not matrix_cores:
        pytest.skip("the kernel that takes any size shares no keys out")
    r, bs, heads, t = 32, 16, 3, 700
    dtype = torch.bfloat16 if matrix_cores else torch.float32
    pages, table, slots = shuffled_pages(t, bs)
    for far in (0, 1, 15, 16, 31, 32, 333, 698, 699):
        rows = torch.zeros(pages * bs, r, dtype=F64)
        rows[slots, 1] = 1.0
        rows[slots[far]] = 0.0
        rows[slots[far], 0] = 5.0
        pool = dev(rows.view(pages, 1, bs, r), dtype)
        q = torch.zeros(1, heads, r, dtype=F64)
        q[..., 0] = 1.0
        out = torch.full((1, heads * r), float("nan"), dtype=dtype, device=DEV)
        common = dict(heads=heads, r=r, dr=0, block_size=bs, window=0, scale=6.0)
        if matrix_cores:
            ops.attend_latent_mfma(out, dev(q.view(1, -1), dtype), pool, table, ints([0, 1]), ints([t]), n_seqs=1, max_count=1,
                                   splits=splits, **common)
        else:
            ops.attend_latent(out, dev(q.view(1, -1), dtype), pool, table, ints([0]), ints([t - 1]), ints([t]), **common)
        got = out.view(heads, r).double().cpu()
        assert float((got[:, 0] - 5.0).abs().max()) < 0.05 and float(got[:, 1:].abs().max()) < 1e-3, f"the row at {far}"


# ------------------------------------------------------------------------------ the stream and the feed-forward
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden", [40, 72, 512, 1100, 2048, 4096, 5000, 77])
def test_a_sum_through_a_norm_and_the_row_as_it_is(dtype, hidden):
    from llmserve.ops import library as ops

    n = 9
    x, y, w = rnd(n, hidden, seed=1), rnd(n, hidden, seed=2, scale=7.0), rnd(hidden, seed=3) + 1
    stream = dev(x)
    out = ops.normed_add_norm(torch.empty((n, hidden), dtype=dtype, device=DEV), stream, None, 0.0, y=dev(y), y_weight=dev(0.3 * w), y_eps=1e-3)
    want = pr.joined(x, y, w, 1e-3, 0.3)
    close(stream, want, torch.float32, "the stream")
    close(out, want, dtype, "what the sublayer reads", loose=0.5)
    alone = ops.normed_add_norm(torch.empty((n, hidden), dtype=dtype, device=DEV), stream, None, 0.0)
    assert torch.equal(alone, stream.to(dtype)) and torch.equal(out, alone)
    rows = ints([4, 4, 0, 8])
    picked = ops.normed_add_norm(torch.empty((4, hidden), dtype=dtype, device=DEV), stream, None, 0.0, rows=rows)
    assert torch.equal(picked, stream.to(dtype)[rows.long()])


def test_a_norm_with_a_factor():
    from llmserve.parts import model  # noqa: F401
    from llmserve.parts.registry import NORMS, BuildContext
    from llmserve.parts.spec import PartSpec

    part = NORMS.build(PartSpec("rmsnorm_streams", {"hidden": 48, "eps": 1e-3, "tensor": "", "multiplier": 0.35}), BuildContext(torch.float32, DEV))
    w, x = rnd(48, seed=1), rnd(5, 48, seed=2)
    part.load({"": dev(w)})
    close(part.forward(dev(x)), 0.35 * pr.rms(x, 1e-3, w), torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,ff", [(64, 96), (44, 30), (128, 512), (72, 56)])
def test_the_gelu_gated_feed_forward_at_every_row_count(dtype, width, ff):
    from llmserve.models.ramolix import _mlp_spec
    from llmserve.parts import model  # noqa: F401
    from llmserve.parts.registry import FEED_FORWARDS, BuildContext

    t = {"gate": rnd(ff, width, seed=30, scale=0.4), "up": rnd(ff, width, seed=31, scale=0.4), "down": rnd(width, ff, seed=32, scale=0.4)}
    h = rnd(200, width, seed=33)
    if dtype == torch.bfloat16:
        h, t = bf16(h), {k: bf16(v) for k, v in t.items()}
    part = FEED_FORWARDS.build(_mlp_spec(width, {"kind": "dense", "ff": ff}), BuildContext(dtype, DEV))
    assert set(part.param_infos()) == set(t)
    part.load({k: dev(v, dtype) for k, v in t.items()})
    for rows in (1, 8, 16, 17, 40, 64, 65, 200):
        close(part.forward(dev(h[:rows], dtype)), pr.gelu_gated(h[:rows], t, ""), dtype, f"{rows} rows", loose=2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_gelu_unit_far_from_zero(dtype):
    """Gates from -40 to 40: nothing overflows, the tails are 0 and the gate itself."""
    from llmserve.ops import library as ops

    for inter in (8, 11, 64):
        gate = torch.linspace(-40, 40, 5 * inter, dtype=F64).view(5, inter)
        up = rnd(5, inter, seed=1)
        gu = torch.cat([gate, up], dim=1).to(dtype)
        out = ops.silu_mul(torch.empty((5, inter), dtype=dtype, device=DEV), gu.to(DEV), gelu=True)
        gu = gu.double()
        close(out, pr.gelu_tanh(gu[:, :inter]) * gu[:, inter:], dtype, f"{inter}", loose=0.5)


# ------------------------------------------------------------------------------ whole models
def write_model(folder, config, seed):
    from safetensors.torch import load_file, save_file

    from llmserve.weights import write_random_model

    # stored in bfloat16, so that both engines and the plain implementation hold the same numbers
    write_random_model(folder, config, seed=seed, dtype=torch.bfloat16, std=0.12, norm_std=0.05)
    tensors = load_file(str(folder / "model.safetensors"))
    g = torch.Generator().manual_seed(seed)
    for name in tensors:
        if name.endswith(".A_log"):  # decays from hardly any to strong
            tensors[name] = (1.5 * torch.randn(tensors[name].shape, generator=g) - 1.0).to(torch.bfloat16)
        if name.endswith(".norm1") or name.endswith(".norm2") or name == "final.norm":
            tensors[name] = (tensors[name].float() * 1.5).to(torch.bfloat16)
        if name.endswith(".q.norm") or name.endswith(".k.norm"):
            tensors[name] = (tensors[name].float() * 1.6).to(torch.bfloat16)
    save_file(tensors, str(folder / "model.safetensors"))
    return {k: v.double() for k, v in tensors.items()}


def position_errors(got, ref, scale):
    d = got.double() - ref.double()
    d = d - d.mean(dim=-1, keepdim=True)
    return d.pow(2).mean(dim=-1).sqrt() / scale


def logits_close(got, ref, dtype, what, noise=None):
    """Per position: the difference of the logits (mean taken off, root mean square over the vocabulary) against the
    root mean square of the logits themselves.  32-bit: every position.  bfloat16: against `noise`, the plain logits
    with nothing but operands of matrix products rounded to bfloat16, which no bfloat16 engine avoids: the median, the upper
    quartile and the worst of the engine's differences stay within three times those of that rounding alone."""
    got, ref = (torch.cat(list(x)) if isinstance(x, (list, tuple)) else x for x in (got, ref))
    scale = ref.double().pow(2).mean().sqrt()
    assert got.shape == ref.shape and torch.isfinite(got).all(), what
    err = position_errors(got, ref, scale)
    worst = int(err.argmax())
    if dtype == torch.float32:
        assert float(err.max()) <= 5e-5, f"{what}: position {worst} is off by {float(err.max()):.2e}"
        return
    floor = position_errors(torch.cat(list(noise)) if isinstance(noise, (list, tuple)) else noise, ref, scale)
    for q in (0.5, 0.75, 1.0):
        a, b = float(err.quantile(q)), float(floor.quantile(q))
        assert a <= 3.0 * b + 2e-3, f"{what}: quantile {q} of the positions is off by {a:.2e}, rounding alone by {b:.2e}"


MODELS = {"small": (SMALL, 8), "small_b": (SMALL_B, 16), "small_c": (SMALL_C, 4), "small_d": (SMALL_D, 16)}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for i, (name, (config, bs)) in enumerate(MODELS.items()):
        folder = tmp_path_factory.mktemp(f"ramolix_{name}")
        out[name] = (folder, config, write_model(folder, config, seed=270 + i), bs)
    return out


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

    runner = ModelRunner.from_folder(folder, EngineConfig(**kwargs))
    runner.storage.poison()  # pages hold NaN until the engine writes them
    for state in runner.storage.state.values():  # and slots until they are taken
        state.fill_(float("nan"))
    return runner


@pytest.mark.parametrize("name", list(MODELS))
def test_the_stream_after_every_layer(models, name):
    from llmserve.engine.batch import build_batch

    folder, config, w, bs = models[name]
    ids = traces.random_ids(config["vocab"], 45, 5)
    want = []
    pr.forward(config, w, ids, collect=want)
    runner = runner_of(folder, dtype="float32", block_size=bs, num_blocks=16, max_num_seqs=2, use_graphs=False)
    runner.add_sequence("a")
    layout = runner.manager.append(["a"], [len(ids)])
    runner.storage.clear_state(layout.fresh_slots)
    batch = build_batch(layout, [ids], [0], runner._uploader, runner.storage)
    model = runner.model
    sources = model.cache_sources()
    x, delta = model.embedding.forward(batch.token_ids), None
    for pos, index in enumerate(model.spec.schedule):
        x, delta = model.blocks[index].forward(x, delta, batch, runner.storage.layer_cache(pos, sources[pos]))
        y = delta.y.double()
        after = x.view(len(ids), -1).double() + y / torch.sqrt((y * y).mean(-1, keepdim=True) + delta.eps) * delta.weight.double()
        close(after, want[pos], torch.float32, f"after layer {pos}")


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(MODELS))
@pytest.mark.parametrize("graphs", [True, False])
def test_every_way_of_cutting_gives_the_plain_logits(models, name, dtype_name, graphs):
    folder, config, w, bs = models[name]
    dtype = getattr(torch, dtype_name)
    seqs = {f"r{i}": traces.random_ids(config["vocab"], n, 300 + i) for i, n in enumerate([67, 1, 30, 41, 2, 75])}
    ref = {rid: pr.forward(config, w, ids) for rid, ids in seqs.items()}
    noise = [pr.forward(config, w, ids, rounded=bf16) for ids in seqs.values()] if dtype == torch.bfloat16 else None
    modes = {"whole": traces.whole(seqs), "decode": traces.prefill_then_decode(seqs, tail=40),
             "portions": traces.portions(seqs), "mixed": traces.mixed(seqs, seed=3, live_max=3)}
    for mode, steps in modes.items():
        pages = -(-traces.tokens_needed(steps, round_to=bs) // bs)
        runner = runner_of(folder, dtype=dtype_name, block_size=bs, num_blocks=pages, max_num_seqs=3, use_graphs=graphs)
        assert runner._use_graphs == graphs  # every part of the model can be captured
        got = run_trace(runner, steps)
        logits_close([got[rid] for rid in seqs], [ref[rid] for rid in seqs], dtype, f"{name} {mode} {dtype_name}", noise)
        assert runner.manager.num_free_slots == 3
        assert all(a.num_free == pages for a in runner.manager.allocators.values())
        if graphs and mode == "decode":
            assert runner._graphs, "steps of single tokens were not replayed from a graph"


@pytest.mark.parametrize("name", ["small", "small_d"])
def test_a_batch_gives_each_request_what_it_gets_alone(models, name):
    folder, config, _w, bs = models[name]
    seqs = {f"b{i}": traces.random_ids(config["vocab"], n, 500 + i) for i, n in enumerate([50, 13, 29])}
    runner = runner_of(folder, dtype="float32", block_size=bs, num_blocks=64, max_num_seqs=3)
    alone = run_trace(runner, traces.portions(seqs))
    together = run_trace(runner, traces.mixed(seqs, seed=9, live_max=3))
    for rid in seqs:
        assert (alone[rid] - together[rid]).abs().max() <= 2e-5 * float(alone[rid].abs().max())


def test_long_decoding_and_the_prompt_of_the_same_tokens_agree(models):
    """280 tokens: whole in one step, and most of them one by one through pages and state; then again on the pages and the
    slot that came back."""
    folder, config, w, bs = models["small_c"]
    ids = traces.random_ids(config["vocab"], 280, 77)
    ref = pr.forward(config, w, ids)
    for graphs in (True, False):
        runner = runner_of(folder, dtype="float32", block_size=bs, num_blocks=-(-280 // bs) + 1, max_num_seqs=1, use_graphs=graphs)
        got = run_trace(runner, traces.prefill_then_decode({"long": ids}, tail=250))
        logits_close(got["long"], ref, torch.float32, "long decoding")
        whole = run_trace(runner, traces.whole({"again": ids}))
        logits_close(whole["again"], ref, torch.float32, "the whole prompt on the pages and the slot that came back")


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
def test_a_long_request_at_matrix_core_sizes(models, dtype_name):
    """650 tokens at sizes the matrix-core kernels take: the prompt in one step and its last tokens one by one (keys shared
    out to several workgroups, several runs of the recurrence), then in portions on what came back."""
    folder, config, w, bs = models["small_d"]
    dtype = getattr(torch, dtype_name)
    ids = traces.random_ids(config["vocab"], 650, 78)
    ref = pr.forward(config, w, ids)
    noise = pr.forward(config, w, ids, rounded=bf16) if dtype == torch.bfloat16 else None
    runner = runner_of(folder, dtype=dtype_name, block_size=bs, num_blocks=-(-650 // bs) + 1, max_num_seqs=1)
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
        ref = pr.forward(config, w, prompt + result.tokens)
        far = 0
        for i, tok in enumerate(result.tokens):
            row = ref[len(prompt) - 1 + i]
            if dtype_name == "float32":  # the plain implementation's own choice, but for a tie within rounding
                far += float(row.max() - row[tok]) > 1e-4 * float(ref.pow(2).mean().sqrt())
            else:
                far += float(row.max() - row[tok]) > 0.1 * float(ref.pow(2).mean().sqrt()) + 1e-3
        assert far == 0
    assert llm.runner.manager.num_free_slots == 3


def test_named_sizes_run_from_the_command_line_entry(capsys):
    from llmserve.cli import main

    assert main(["--model", "ramolix-tiny", "--random-weights", "--max-new-tokens", "5", "--dtype", "float32"]) == 0
    assert "decode=" in capsys.readouterr().out


def drawn_config(seed: int) -> tuple[dict, int]:
    """A configuration drawn at random from what config.json allows: the three mixers in any order, with feed-forwards or
    without, latents of a layer's own or an earlier layer's, sizes from 1 or 2 up and beyond 64, windows from one key up or
    none, rotations over all, a part or nothing of a head, stretched or not; and a page size."""
    rng = random.Random(seed)
    layers, owners = [], []
    for i in range(rng.randint(3, 6)):
        ff = rng.choice([None, 8, 30, 96])
        kind = rng.random()
        if kind < 0.4:
            heads, groups = rng.choice([(1, 1), (4, 2), (6, 1), (6, 6), (9, 3)])
            vdim, parts = rng.choice([4, 7, 16, 32, 48]), rng.choice([1, heads, 2])
            parts = parts if heads * vdim % parts == 0 else 1
            layers.append(space(ff, heads=heads, groups=groups, vdim=vdim, state=rng.choice([2, 9, 16, 48, 128]), conv=rng.choice([1, 2, 4, 6]),
                                norm_groups=parts))
        elif kind < 0.7:
            kv, dim = rng.choice([1, 2, 3]), rng.choice([4, 10, 16, 32, 48, 64])
            rot = {"base": rng.choice([10.0, 10000.0, 1e6]), "dims": rng.choice([dim, dim // 2 // 2 * 2, 2, 0])}
            if rng.random() < 0.5:
                rot["scaling"] = dict(STRETCH, factor=rng.choice([2.0, 8.0]), original=rng.choice([32, 256]))
            layers.append(attention(ff, heads=kv * rng.choice([1, 2, 3]), kv_heads=kv, dim=dim, scale=rng.choice([0.3, 1.0, 2.0]) / math.sqrt(dim),
                                    rot=rot, mask=rng.choice([None, {"size": 1}, {"size": 5}, {"size": 16}, {"size": 33}, {"size": 100}])))
        else:
            sizes = dict(heads=rng.randint(1, 5), dim=rng.choice([4, 8, 16, 20, 32]), vdim=rng.choice([4, 8, 16, 40]), scale=rng.choice([0.2, 0.5, 1.0]))
            if owners and rng.random() < 0.5:
                src = rng.choice(owners)
                layers.append(latent(ff, kv_rank=layers[src]["mixer"]["kv_rank"], kv_from=src, **sizes))
            else:
                owners.append(i)
                layers.append(latent(ff, kv_rank=rng.choice([8, 16, 30, 48]), **sizes))
    return config_of(layers, width=rng.choice([40, 64, 72, 100]), vocab=rng.choice([61, 128, 257]), eps=rng.choice([1e-6, 1e-5]),
                     embedding=rng.choice([1.0, 4.0, 12.5]), mult=rng.choice([0.2, 0.7, 1.0])), rng.choice([4, 8, 16])


@pytest.mark.parametrize("seed", list(range(12)))
def test_configurations_drawn_at_random(tmp_path, seed):
    config, bs = drawn_config(seed)
    w = write_model(tmp_path, config, seed=1900 + seed)
    seqs = {f"q{i}": traces.random_ids(config["vocab"], n, 40 * seed + i) for i, n in enumerate([90, 3, 47, 160, 18])}
    ref = {rid: pr.forward(config, w, ids) for rid, ids in seqs.items()}
    noise = [pr.forward(config, w, ids, rounded=bf16) for ids in seqs.values()]
    for dtype_name in ("float32", "bfloat16"):
        steps = traces.mixed(seqs, seed=seed, live_max=3, tail=30)
        pages = -(-traces.tokens_needed(steps, round_to=bs) // bs)
        runner = runner_of(tmp_path, dtype=dtype_name, block_size=bs, num_blocks=pages, max_num_seqs=3)
        got = run_trace(runner, steps)
        logits_close([got[rid] for rid in seqs], [ref[rid] for rid in seqs], getattr(torch, dtype_name),
                     f"seed {seed} {dtype_name}: {config['layers']}", noise)
        assert runner.manager.num_free_slots == 3
        assert all(a.num_free == pages for a in runner.manager.allocators.values())
