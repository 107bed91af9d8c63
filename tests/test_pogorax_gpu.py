"""Pogorax on the GPU against the plain implementation (``plain_pogorax``): every mechanism's kernels alone and as a one-layer
model, then the engine under schedules (whole, token by token, portions down to two tokens, unequal requests in one batch, pages
and state slots used again, long decoding) and greedy generation through ``LLM`` and the command line.  Configurations and weights
are the tests' own; where random weights would hide a fault (a key at a chunk's edge or far away, a decay near 0 or 1, a gate, a
branch that outweighs the other), inputs are made so that it shows."""
import functools
import json
import math
import os
import tempfile
import types

import numpy as np
import pytest
import torch

import plain_pogorax as pp
from helpers import check

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
TD = {"float32": torch.float32, "bfloat16": torch.bfloat16}
_keep = []


def T(a):
    return torch.as_tensor(np.asarray(a), dtype=torch.float64)


def close(got, want, dtype, what, scale=None):
    got, want = torch.as_tensor(got).double().cpu(), T(want)
    bound = (2e-5 if dtype == "float32" else 2e-2) * (float(want.abs().max()) if scale is None else scale)
    err = float((got - want.reshape(got.shape)).abs().max())
    assert err <= bound, f"{what}: {err:.3e} > {bound:.3e}"


def mostly(got, ref, dtype, what, moves=None):
    """Every row against the plain logits: 32-bit to rounding; bfloat16 to a quarter of the spread everywhere and to a
    tenth at nine rows in ten (the tests' models are narrow).  ``moves``: how far the plain logits of every row move themselves when
    weights are off by their last place (a head's output that is a small difference of large terms is brought to unit RMS all the same):
    bfloat16 rows are allowed three times that where it is more."""
    ref = T(ref)
    if dtype == "float32":
        return check(got, ref, dtype, what)
    got = torch.as_tensor(got).double().reshape(ref.shape)
    err = (got - ref).abs().reshape(len(ref), -1).max(dim=1).values / float(ref.std())
    if moves is not None:
        err = err * torch.clamp(0.08 / T(moves), max=1.0)
    assert float(err.max()) <= 0.25, f"{what}: row {int(err.argmax())} is off by {float(err.max()):.3f} of the spread"
    over = int((err > 0.1).sum())
    assert over <= max(1, len(err) // 10), f"{what}: {over} of {len(err)} rows are off by more than a tenth of the spread"


def rnd(shape, seed, dtype, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(shape, generator=g) * scale).to(TD[dtype])


def step_of(ctx, qn, gpu, slots=None, page=8):
    """The index arrays of a step whose sequences have ``ctx`` tokens after it and bring ``qn`` of them."""
    cu = np.concatenate([[0], np.cumsum(qn)]).astype(np.int32)
    pos = np.concatenate([np.arange(c - n, c) for c, n in zip(ctx, qn)]).astype(np.int32)
    seq = np.concatenate([[i] * n for i, n in enumerate(qn)]).astype(np.int32)
    dec = [i for i, n in enumerate(qn) if n == 1]
    pre = [i for i, n in enumerate(qn) if n > 1]
    dev = lambda a: torch.tensor(np.asarray(a), dtype=torch.int32, device=gpu)
    return types.SimpleNamespace(
        positions=dev(pos), seq_of_token=dev(seq), cu_q=dev(cu), context_lens=dev(ctx), decode_seqs=dev(dec), prefill_seqs=dev(pre),
        state_slots=dev(slots if slots is not None else list(range(len(ctx)))), num_seqs=len(ctx), num_tokens=int(cu[-1]),
        n_decode=len(dec), n_prefill=len(pre), max_decode_context=max([ctx[i] for i in dec], default=0), max_q_len=max(qn),
        max_prefill_q=max([qn[i] for i in pre], default=0), min_prefill_prefix=min([ctx[i] - qn[i] for i in pre], default=0),
        page_size=page)


def feed(lens, cuts, slots, gpu, run):
    """Feeds sequences of ``lens`` tokens in portions: step k brings ``cuts[i][k]`` tokens of sequence i.  ``run(pieces, step)`` gets
    [(sequence, begin, end), ..] and returns rows; the rows of every sequence come back in one piece each."""
    got, fed = [[] for _ in lens], [0] * len(lens)
    for k in range(max(len(c) for c in cuts)):
        live = [i for i in range(len(lens)) if k < len(cuts[i])]
        qn = [cuts[i][k] for i in live]
        pieces = [(i, fed[i], fed[i] + n) for i, n in zip(live, qn)]
        out = run(pieces, step_of([b for _, _, b in pieces], qn, gpu, slots=[slots[i] for i in live])).cpu()
        at = 0
        for i, n in zip(live, qn):
            got[i].append(out[at: at + n])
            at += n
            fed[i] += n
    assert fed == list(lens)
    return [torch.cat(g) for g in got]


CUTS = ([333, 6, 150], [[1, 1, 200, 2, 65, 64], [2, 1, 1, 2], [130, 7, 1, 12]])   # lengths; portions per step
SLOTS = [3, 0, 4]


# ---- norms -----------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden", [36, 37, 64, 2056, 5000, 9000])
def test_branches_brought_to_unit_rms_in_front_of_a_stream(gpu, dtype, hidden):
    """Two branches of very different size, as tensors and as slices, one alone; chosen rows with the stream left as it is; the
    stream normed by itself."""
    from prelude_amd.ops import kernels as K
    n, g = 5, torch.Generator().manual_seed(1)
    x = torch.randn((n, hidden), generator=g) * 3
    a, b = rnd((n, hidden), 2, dtype, 50.0), rnd((n, hidden), 3, dtype, 0.02)
    parts = torch.randn((3, n, hidden), generator=g)
    wa, wb, w = (1 + 0.3 * torch.randn(hidden, generator=g) for _ in range(3))
    eps, beps = 1e-5, 1e-4
    unit = lambda y, wt: pp.rms_unit(y.double().numpy(), beps) * wt.double().numpy()
    norm = lambda s: pp.rms_unit(s, eps) * w.double().numpy()
    dev = lambda t: t.to(gpu)
    sl = K.SliceSums(dev(parts), TD[dtype])
    cases = [("two tensors", [dev(a), dev(b)], [wa, wb], [0.5, 0.5], 0.5 * unit(a, wa) + 0.5 * unit(b, wb)),
             ("a tensor and slices", [dev(a), sl], [wa, wb], [1.0, -2.0], unit(a, wa) - 2.0 * unit(parts.double().sum(0), wb)),
             ("slices and a tensor", [sl, dev(b)], [wb, wa], [0.25, 1.0], 0.25 * unit(parts.double().sum(0), wb) + unit(b, wa)),
             ("one", [dev(a)], [wa], [0.5], 0.5 * unit(a, wa))]
    for what, ys, ws, cs, want in cases:
        nb = K.NormedBranches(ys, [dev(v) for v in ws], cs, beps)
        s = dev(x.clone())
        total = x.double().numpy() + want
        rows = torch.tensor([3, 0, 3], dtype=torch.int32, device=gpu)
        close(K.branches_norm_step(nb, s, dev(w), eps, rows=rows), norm(total)[[3, 0, 3]], dtype, f"{what}: chosen rows")
        assert torch.equal(s.cpu(), x), "read only"
        close(K.branches_norm_step(nb, s, dev(w), eps), norm(total), dtype, what)
        close(s, total, "float32", f"{what}: the stream took them")
        close(nb.materialize(), want, "float32", f"{what}: the sum alone")
    s = dev(x.clone())
    close(K.rmsnorm_wide(None, dev(w), eps, residual=s, out_dtype=TD[dtype]), norm(x.double().numpy()), dtype, "the stream alone")
    assert torch.equal(s.cpu(), x)
    y = rnd((n, hidden), 4, dtype)
    close(K.rmsnorm_wide(dev(y), dev(w), eps, residual=s), norm(x.double().numpy() + y.double().numpy()), dtype, "with what waits")
    close(s, x.double() + y.double(), "float32", "the stream took it")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,groups", [(36, 3), (37, 1), (256, 2), (4096, 8), (1536, 1), (15, 5), (5000, 1)])
def test_gate_in_front_of_a_norm_in_groups(gpu, dtype, width, groups):
    from prelude_amd.ops import kernels as K
    n, g = 7, torch.Generator().manual_seed(5)
    y, w = torch.randn((n, width), generator=g), 1 + 0.3 * torch.randn(width, generator=g)
    y[:, : width // groups] *= 100.0                               # one group outweighs the others: each has its own norm
    wide = rnd((n, width + 24), 6, dtype, 3.0)
    out = torch.full((n, width + 16), 9.0, dtype=TD[dtype], device=gpu)
    u = y.double().numpy() * pp.silu(wide[:, 8: 8 + width].double().numpy())
    want = 0.5 * pp.rms_unit(u.reshape(n, groups, -1), 1e-5).reshape(n, width) * w.double().numpy()
    K.gated_group_norm(y.to(gpu), wide.to(gpu)[:, 8: 8 + width], w.to(gpu), groups, 1e-5, out[:, 8: 8 + width], 0.5)
    close(out[:, 8: 8 + width], want, dtype, "columns of wider rows")
    assert (out[:, :8] == 9.0).all() and (out[:, 8 + width:] == 9.0).all(), "nothing beside them"


@pytest.mark.parametrize("dtype", DTYPES)
def test_heads_over_a_denominator_and_their_norm(gpu, dtype):
    """The denominator is the larger of |n.q| and the floor, either way round; every head has weights of its own."""
    from prelude_amd.ops import kernels as K
    n, H, e, g = 6, 3, 20, torch.Generator().manual_seed(7)
    o, den = torch.randn((n, H, e), generator=g), torch.randn((n, H), generator=g) * 3
    floor = torch.exp(torch.randn((n, H), generator=g))
    o[0] *= 1e-4                                                   # eps counts behind the division: the head's own size does too
    w, gate = 1 + 0.3 * torch.randn(H * e, generator=g), rnd((n, H * e + 4), 8, dtype, 2.0)
    u = o.double().numpy() / (np.maximum(np.abs(den.numpy()), floor.numpy()) + 1e-6)[..., None]
    want = pp.rms_unit(u, 1e-5).reshape(n, -1) * w.numpy() * pp.sigmoid(gate[:, 4:].double().numpy())
    got = K.head_norm_gate(o.to(gpu), gate.to(gpu)[:, 4:], w.to(gpu), 1e-5, "sigmoid", None, 1.0, den.to(gpu), floor.to(gpu), 1e-6)
    close(got, want, dtype, "over a denominator")


# ---- convolution ---------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C,taps,act,biases", [(40, 4, "silu", (False, True)), (15, 4, None, (True, True)), (64, 4, None, (True, True)),
                                               (24, 3, "silu", (True, False)), (7, 1, "silu", (False, True)), (512, 2, None, (False, False)),
                                               (72, 6, "silu", (True, True))])
def test_short_convolution_across_cuts(gpu, dtype, C, taps, act, biases):
    """With a bias on the inputs (which the zeros before a sequence's start do not have) and one on the sum, out of wider rows;
    more than 512 tokens in one step beside single tokens, so that runs of tokens take every path."""
    from prelude_amd.ops import kernels as K
    g = torch.Generator().manual_seed(10)
    w = torch.randn((C, taps), generator=g)
    ib, b = (torch.randn(C, generator=g) if on else None for on in biases)
    lens, cuts = [700, 6, 150], [[1, 1, 560, 2, 72, 64], [2, 1, 1, 2], [130, 7, 1, 12]]
    seqs = [rnd((n, C + 16), 11 + n, dtype) for n in lens]
    state = torch.full((5, taps - 1, C), 7.0, device=gpu) if taps > 1 else None
    if taps > 1:
        state[SLOTS] = 0.0
    dev = lambda t: None if t is None else t.to(gpu)
    got = feed(lens, cuts, SLOTS, gpu, lambda pieces, st: K.time_conv(torch.cat([seqs[i][a:z] for i, a, z in pieces]).to(gpu)[:, 8: 8 + C],
                                                                      w.t().contiguous().to(gpu), state, st, dev(ib), dev(b), act))
    for i, s in enumerate(seqs):
        x = s[:, 8: 8 + C].double().numpy() + (0.0 if ib is None else ib.double().numpy())
        want = pp.short_conv(x, w.double().numpy(), 0.0 if b is None else b.double().numpy())
        close(got[i], pp.silu(want) if act else want, dtype, f"sequence {i}")
        if taps > 1:
            tail = np.concatenate([np.zeros((taps - 1, C)), x])[-(taps - 1):]
            close(state[SLOTS[i]], tail, "float32", f"what sequence {i} carries")
    if taps > 1:
        assert (state[[1, 2]] == 7.0).all(), "another request's slot is left alone"


# ---- recurrences with one decay a token -------------------------------------------------------------------------------------
@pytest.mark.parametrize("chunked", [True, False])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,groups,d,e", [(6, 3, 24, 16), (4, 1, 128, 64), (3, 3, 7, 5), (8, 2, 48, 72), (2, 2, 200, 136), (2, 1, 256, 8)])
def test_ssd_recurrence_across_cuts(gpu, dtype, heads, groups, d, e, chunked, monkeypatch):
    """Portions (in chunks on the matrix cores in bfloat16 where the widths allow it) beside single tokens; heads that forget
    everything at once, heads that forget nothing, and steps that jump between both inside a chunk."""
    from prelude_amd.ops import kernels as K
    if dtype == "float32" and not chunked:
        pytest.skip("the 32-bit engine has one path")
    monkeypatch.setattr(K, "DECAY_SCAN_CHUNKED", chunked)
    g = torch.Generator().manual_seed(20)
    a_log, bias, skip = torch.randn(heads, generator=g), torch.randn(heads, generator=g) - 2, torch.randn(heads, generator=g)
    a_log[0], a_log[-1] = 6.0, -12.0
    lens, cuts = CUTS
    gn, vv = groups * d, heads * e
    width = vv + 2 * gn
    seqs, steps = [rnd((n, width), 21 + n, dtype) for n in lens], [rnd((n, heads + 8), 31 + n, dtype) for n in lens]
    for s in steps:
        s[5::7, 8:] += 12.0                                         # long steps: nearly everything before them is gone
    state = torch.full((5, heads, d, e), 3.0, device=gpu)
    state[SLOTS] = 0.0
    dev = lambda t: t.to(gpu)

    def run(pieces, st):
        p, z = (torch.cat([x[i][a:b] for i, a, b in pieces]).to(gpu) for x in (seqs, steps))
        return K.ssd_scan(p, vv + gn, vv, 0, z[:, 8:], dev(bias), dev(a_log), dev(skip), state, st, heads, groups, d, e)
    got = feed(lens, cuts, SLOTS, gpu, run)
    tol = 1.0 if dtype == "float32" else 2.0     # inputs are what they are in both formats, everything behind them is 32-bit
    for i, n in enumerate(lens):
        x = seqs[i].double().numpy()
        B, C = (np.repeat(v.reshape(n, groups, d), heads // groups, axis=1) for v in (x[:, vv: vv + gn], x[:, vv + gn:]))
        dt = pp.softplus(steps[i][:, 8:].double().numpy() + bias.double().numpy())
        y, S = pp.ssd_recurrence(C, B, x[:, :vv].reshape(n, heads, e), dt, np.exp(a_log.double().numpy()), skip.double().numpy())
        for h in range(heads):                                      # head by head: their sizes differ
            close(got[i][:, h], y[:, h], "float32", f"sequence {i} head {h}", scale=tol * max(1.0, float(np.abs(y[:, h]).max())))
            close(state[SLOTS[i], h], S[h], "float32", f"the state of sequence {i} head {h}", scale=tol * max(1e-3, float(np.abs(S[h]).max())))
    assert (state[[1, 2]] == 3.0).all(), "another request's slot is left alone"


@pytest.mark.parametrize("chunked", [True, False])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,d,e,cap", [(3, 16, 24, 9.0), (2, 64, 128, 15.0), (1, 5, 7, 3.0), (4, 128, 32, 20.0), (2, 200, 136, 12.0), (1, 256, 264, 30.0)])
def test_mlstm_recurrence_across_cuts(gpu, dtype, heads, d, e, cap, chunked, monkeypatch):
    """Gates that run into their cap on either side, input gates that jump far above everything before (the running maximum
    moves) and far below (the floor e^-m is the larger part of the denominator), a forget gate near 1 over hundreds of tokens."""
    from prelude_amd.ops import kernels as K
    if dtype == "float32" and not chunked:
        pytest.skip("the 32-bit engine has one path")
    monkeypatch.setattr(K, "DECAY_SCAN_CHUNKED", chunked)
    g = torch.Generator().manual_seed(40)
    ib, fb = torch.randn(heads, generator=g), 4 + torch.randn(heads, generator=g)
    fb[-1] = 20.0
    lens, cuts = CUTS
    qk, vv = heads * d, heads * e
    gates = 2 * qk + vv
    width = (8 + gates + 2 * heads + 7) // 8 * 8
    seqs = [rnd((n, width), 41 + n, dtype) for n in lens]
    for s in seqs:
        s[:, 8 + gates: 8 + gates + heads] *= 3.0
        s[40::50, 8 + gates: 8 + gates + heads] = 3.0 * cap         # far above
        s[20:30, 8 + gates: 8 + gates + heads] = -3.0 * cap         # far below
        s[60::90, 8 + gates + heads: 8 + gates + 2 * heads] = -3.0 * cap
    s_state, n_state = torch.full((5, heads, d, e), 3.0, device=gpu), torch.full((5, heads, d), 3.0, device=gpu)
    m_state = torch.full((5, heads, K.mlstm_max_copies(e)), 3.0, device=gpu)
    for t in (s_state, n_state, m_state):
        t[SLOTS] = 0.0
    dev = lambda t: t.to(gpu)

    def run(pieces, st):
        p = torch.cat([seqs[i][a:b] for i, a, b in pieces]).to(gpu)
        o, den, floor = K.mlstm_scan(p, 8, 8 + qk, 8 + 2 * qk, 8 + gates, 8 + gates + heads, dev(ib), dev(fb), cap, s_state, n_state, m_state, st, heads,
                                     d, e, d ** -0.5)
        return torch.cat([o.reshape(len(p), -1), den, floor], dim=1)
    got = feed(lens, cuts, SLOTS, gpu, run)
    tol = 1.0 if dtype == "float32" else 2.0
    for i, n in enumerate(lens):
        x = seqs[i].double().numpy()[:, 8:]
        ig = cap * np.tanh((x[:, gates: gates + heads] + ib.double().numpy()) / cap)
        fg = pp.log_sigmoid(cap * np.tanh((x[:, gates + heads: gates + 2 * heads] + fb.double().numpy()) / cap))
        q = x[:, :qk].reshape(n, heads, d) * d ** -0.5
        want, (S, nn, m) = pp.mlstm_recurrence(q, x[:, qk: 2 * qk].reshape(n, heads, d), x[:, 2 * qk: gates].reshape(n, heads, e), ig, fg)
        out = got[i].double().numpy()
        o, den, floor = out[:, :vv].reshape(n, heads, e), out[:, vv: vv + heads], out[:, vv + heads:]
        full = o / (np.maximum(np.abs(den), floor) + 1e-6)[..., None]
        for h in range(heads):
            # a denominator that is a small difference of large terms magnifies the rounding of both sums: row by row, by how much
            size = np.abs(want[:, h]).max() * np.ones(n)
            bound = tol * 3e-5 * np.maximum(size, 1.0) * (1.0 + np.sqrt(n) / np.maximum(np.abs(den[:, h]), floor[:, h]))
            err = np.abs(full[:, h] - want[:, h]).max(axis=1)
            assert (err <= bound).all(), f"sequence {i} head {h} token {int((err / bound).argmax())}: {err.max():.3e}"
        close(m_state[SLOTS[i]], np.repeat(m[:, None], m_state.shape[2], axis=1), "float32", f"the running maximum of sequence {i}", scale=tol * cap)
        close(s_state[SLOTS[i]], S, "float32", f"S of sequence {i}", scale=2 * tol * float(np.abs(S).max()))
        close(n_state[SLOTS[i]], nn, "float32", f"n of sequence {i}", scale=2 * tol * float(np.abs(nn).max()))
    assert all((t[[1, 2]] == 3.0).all() for t in (s_state, n_state, m_state)), "another request's slot is left alone"


def test_long_portion_of_gates_and_a_maximum_that_holds(gpu):
    """2,500 tokens in one step (several blocks of the gates' scan): one input gate far above all others near the start, a forget
    gate of almost 1: the maximum it left decides at every later token."""
    from prelude_amd.ops import kernels as K
    heads, d, e, n, cap = 2, 16, 16, 2500, 15.0
    p = rnd((n, 4 * heads * d), 45, "float32")
    gates = 3 * heads * d
    p[3, gates: gates + heads] = 100.0
    ib, fb = torch.zeros(heads), torch.full((heads,), 30.0)
    z = p.double().numpy()
    ig = cap * np.tanh(z[:, gates: gates + heads] / cap)
    fg = pp.log_sigmoid(cap * np.tanh((z[:, gates + heads: gates + 2 * heads] + 30.0) / cap))
    q, k, v = (z[:, j * heads * d: (j + 1) * heads * d].reshape(n, heads, d) for j in range(3))
    _, (S, nn, m) = pp.mlstm_recurrence(q * d ** -0.5, k, v, ig, fg)
    for dtype in DTYPES:
        st = [torch.zeros((1, heads, d, e), device=gpu), torch.zeros((1, heads, d), device=gpu), torch.zeros((1, heads, K.mlstm_max_copies(e)), device=gpu)]
        x = p.to(TD[dtype])
        _, _, floor = K.mlstm_scan(x.to(gpu), 0, heads * d, 2 * heads * d, gates, gates + heads, ib.to(gpu), fb.to(gpu), cap, *st, step_of([n], [n], gpu), heads, d, e,
                                   d ** -0.5)
        tol = 1e-4 if dtype == "float32" else 2e-2
        assert float((st[2][0, :, 0].cpu().double() - T(m)).abs().max()) <= tol
        assert float((floor[-1].cpu().double() - torch.exp(-T(m))).abs().max()) <= tol * float(torch.exp(-T(m)).max())


# ---- a recurrence on every channel ------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,blocks", [(48, 3), (64, 1), (15, 5), (320, 4), (136, 2), (72, 1), (592, 2), (328, 1)])
def test_linear_recurrent_unit_across_cuts(gpu, dtype, width, blocks):
    """Channels that forget nothing (a = 1 to rounding, where 1 - a^2 must not be taken as a difference), channels that forget
    everything, the other branch out of wider rows with its bias."""
    from prelude_amd.ops import kernels as K
    g = torch.Generator().manual_seed(50)
    size = width // blocks
    wr, wi = (rnd((blocks, size, size), 51 + k, dtype, size ** -0.5) for k in range(2))
    br, bi, yb = (torch.randn(width, generator=g) for _ in range(3))
    lam = torch.randn(width, generator=g) - 2
    lam[0], lam[1] = -16.0, 8.0
    rate = (8.0 * torch.nn.functional.softplus(lam.double())).float()
    lens, cuts = CUTS
    us, ys = [rnd((n, width), 53 + n, dtype) for n in lens], [rnd((n, width + 5), 63 + n, dtype) for n in lens]
    state = torch.full((5, width), 3.0, device=gpu)
    state[SLOTS] = 0.0
    dev = lambda t: t.to(gpu)

    def run(pieces, st):
        u, y = (torch.cat([x[i][a:b] for i, a, b in pieces]).to(gpu) for x in (us, ys))
        return K.lru_scan(u, dev(wr), dev(wi), dev(br), dev(bi), dev(rate), state, y[:, 5:], dev(yb), st)
    got = feed(lens, cuts, SLOTS, gpu, run)
    for i in range(3):
        u = us[i].double().numpy()
        gate = lambda w, b: pp.block_gate(u, w.double().numpy(), b.double().numpy().reshape(blocks, size))
        S, end = pp.lru_recurrence(u, gate(wr, br), gate(wi, bi), lam.double().numpy())
        close(got[i], S * pp.gelu_tanh(ys[i][:, 5:].double().numpy() + yb.double().numpy()), dtype, f"sequence {i}")
        # channel by channel: the state of one that forgets nothing is small, and must be right by its own size
        err = (state[SLOTS[i]].cpu().double() - T(end)).abs() / (T(np.abs(S).max(axis=0)) + 1e-12)
        assert float(err.max()) <= (4e-5 if dtype == "float32" else 1e-4), f"the state of sequence {i}: channel {int(err.argmax())} {float(err.max()):.2e}"
    assert (state[[1, 2]] == 3.0).all(), "another request's slot is left alone"


# ---- attention in chunks, with a gate per column ------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nh,nkv,hd,vd,rot,page", [(4, 2, 16, 24, 8, 8), (6, 1, 64, 64, 64, 16), (3, 3, 6, 10, 2, 8), (2, 1, 130, 7, 0, 16)])
def test_rotated_heads_over_their_own_root_mean_square(gpu, dtype, nh, nkv, hd, vd, rot, page):
    from prelude_amd.ops import kernels as K
    n, base, off, eps = 21, 777.0, 5, 1e-2                        # a large eps: its place shows
    nq, nk, nv = nh * hd, nkv * hd, nkv * vd
    p = rnd((n, off + nq + nk + nv + 3), 11, dtype)
    p[:, off: off + hd] *= 0.02
    freq = torch.tensor([base ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=torch.float64).float() if rot else None
    pos = list(range(100, 100 + n))
    x = p.double().numpy()[:, off:]
    q, k, v = x[:, :nq].reshape(n, nh, hd), x[:, nq: nq + nk].reshape(n, nkv, hd), x[:, nq + nk: nq + nk + nv].reshape(n, nkv, vd)
    if rot:
        q, k = pp.rotate_pairs(q, pos, rot, base), pp.rotate_pairs(k, pos, rot, base)
    q, k = pp.rms_unit(q, eps), pp.rms_unit(k, eps)
    pages = -(-n // page)
    perm = torch.randperm(pages, generator=torch.Generator().manual_seed(12)).tolist()
    slots = torch.tensor([perm[i // page] * page + i % page for i in range(n)], dtype=torch.int32, device=gpu)
    kc, vc = torch.zeros((pages, nkv, page, hd), dtype=TD[dtype], device=gpu), torch.zeros((pages, nkv, vd, page), dtype=TD[dtype], device=gpu)
    out = K.qkv_rope_prepare(p.to(gpu), off, off + nq, off + nq + nk, None if freq is None else freq.to(gpu),
                             torch.tensor(pos, dtype=torch.int32, device=gpu), slots, kc, vc, nh, nkv, nkv, hd, vd, rot, True, unit_eps=eps)
    close(out, q, dtype, "queries")
    close(torch.cat([kc[perm[j]].transpose(0, 1) for j in range(pages)])[:n], k, dtype, "keys")
    close(torch.cat([vc[perm[j]].permute(2, 0, 1) for j in range(pages)])[:n], v, dtype, "values")


CHUNKED = [  # heads, key heads, key width, value width, chunk, page
    (4, 1, 64, 128, 80, 16), (4, 2, 16, 24, 20, 8), (8, 2, 128, 128, 100, 16), (6, 3, 32, 64, 33, 32), (20, 1, 40, 12, 64, 16), (3, 3, 64, 64, 1, 8),
    (8, 4, 64, 64, 2, 8), (34, 2, 48, 36, 128, 16), (4, 2, 96, 96, 0, 16), (2, 1, 264, 100, 50, 64), (3, 3, 6, 10, 7, 4)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nh,nk,kd,vd,chunk,page", CHUNKED)
def test_attention_inside_chunks_with_a_gate(gpu, dtype, nh, nk, kd, vd, chunk, page):
    """Portions (a whole prompt over several tiles and chunks, one behind a prefix that ends inside a chunk, two tokens across a
    chunk's edge) beside single tokens at a chunk's first, second and last place, through shuffled pages whose other places hold large
    numbers; the first key of the last query's chunk, the key in front of it, and one far back are made to stand out."""
    from prelude_amd.ops import kernels as K
    C = chunk or 100
    ctx = [3 * C + C // 2 + 40, 2 * C + 30, 2 * C + 1, 4 * C + 1, 4 * C + 2, 5 * C, 1]
    qn = [ctx[0], min(33, ctx[1] - 1), 2, 1, 1, 1, 1]
    step = step_of(ctx, qn, gpu, page=page)
    g = torch.Generator().manual_seed(20)
    scale = kd ** -0.5
    need = [-(-c // page) for c in ctx]
    perm = torch.randperm(sum(need) + 2, generator=g).tolist()
    kc = torch.full((len(perm), nk, page, kd), 30.0, dtype=TD[dtype])
    vc = torch.full((len(perm), nk, vd, page), -30.0, dtype=TD[dtype])
    table = torch.full((len(ctx), max(need)), perm[-1], dtype=torch.int32)
    total = sum(qn)
    gates = rnd((total, nh * vd + 8), 25, dtype, 2.0)
    qs, wants, at, row = [], [], 0, 0
    for s, (c, n) in enumerate(zip(ctx, qn)):
        k, v = torch.randn((c, nk, kd), generator=g), torch.randn((c, nk, vd), generator=g).to(TD[dtype])
        q = torch.randn((n, nh, kd), generator=g).to(TD[dtype])
        last, first = q[-1].float(), (c - 1) // C * C
        for key in {first, first - 1, c // 5}:
            if 0 <= key < c:
                for a in range(nk):
                    k[key, a] = 6.0 * last[a * (nh // nk)] / last[a * (nh // nk)].norm() / scale ** 0.5
        k = k.to(TD[dtype])
        for j in range(need[s]):
            pg = perm[at]
            at += 1
            if chunk and (j + 1) * page <= (c - n) // chunk * chunk:    # wholly before the first query's chunk: given back
                table[s, j] = -1
                continue
            table[s, j] = pg
            m = min(page, c - j * page)
            kc[pg, :, :m] = k[j * page: j * page + m].transpose(0, 1)
            vc[pg, :, :, :m] = v[j * page: j * page + m].permute(1, 2, 0)
        qs.append(q)
        see = pp.visible(c, chunk or None)[c - n:]
        kk, vv, qq = k.double().numpy(), v.double().numpy(), q.double().numpy()
        o = np.stack([pp.softmax_sum(qq[:, a] @ kk[:, a // (nh // nk)].T * scale, see, vv[:, a // (nh // nk)]) for a in range(nh)], axis=1)
        wants.append(o.reshape(n, nh * vd) * pp.sigmoid(gates[row: row + n, 8:].double().numpy()))
        row += n
    group, q, want = types.SimpleNamespace(block_table=table.to(gpu)), torch.cat(qs).to(gpu), np.concatenate(wants)
    kc, vc, gate = kc.to(gpu), vc.to(gpu), gates.to(gpu)[:, 8:]
    size = max(1.0, float(np.abs(want).max()))
    got = K.attention_masked(q, kc, vc, group, step, 0, 0, scale, gate=gate, chunk=chunk)
    close(got, want, dtype, "masked", scale=size)
    if dtype == "bfloat16" and K.attention_wide_supported(kd, vd, page):
        wide = torch.full((total, nh * vd + 12), 5.0, dtype=torch.bfloat16, device=gpu)
        got = K.attention_wide(q, kc, vc, group, step, 0, scale, out=wide[:, 4: 4 + nh * vd], chunk=chunk, gate=gate)
        close(got, want, dtype, "any widths", scale=size)
        assert (wide[:, :4] == 5.0).all() and (wide[:, 4 + nh * vd:] == 5.0).all(), "nothing beside the heads"
        singles = [i for i, n in enumerate(qn) if n == 1]
        st1 = step_of([ctx[i] for i in singles], [1] * len(singles), gpu, page=page)
        rows = [int(sum(qn[:i])) for i in singles]
        for fn, kw in ((K.attention_wide, {}), (K.attention_masked, {"keep_first": 0})):
            got = fn(q[rows].contiguous(), kc, vc, types.SimpleNamespace(block_table=table[singles].to(gpu)), st1, 0, scale=scale, chunk=chunk,
                     gate=gate[rows].contiguous(), **kw)
            close(got, want[rows], dtype, f"single tokens alone, {fn.__name__}", scale=size)


# ---- one-layer models ----------------------------------------------------------------------------------------------------
def write_model(cfg, w):
    from prelude_amd.weights import write_safetensors
    tmp = tempfile.TemporaryDirectory(prefix="prelude_amd_test_pogorax_")
    _keep.append(tmp)
    with open(os.path.join(tmp.name, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(tmp.name, "model.safetensors"), {k: torch.as_tensor(v).to(torch.bfloat16) for k, v in w.items()})
    return tmp.name


def run_cut(path, dtype, toks, cuts, page=8, max_tokens=512):
    """Logits of every position, the prompt fed in portions of ``cuts`` tokens and the rest one by one."""
    from prelude_amd.trace import TraceRunner
    r = TraceRunner(path, dtype, max_tokens, page_size=page, state_slots=1)
    outs, i = [], 0
    for n in list(cuts) + [1] * (len(toks) - sum(cuts)):
        outs.append(r.step([{"id": 0, "tokens": toks[i:i + n], "want": list(range(n))}]))
        i += n
    return np.concatenate(outs)


def tokens(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], size=n).tolist()


ONE_LAYER = [(pp.parallel_layer, {}), (pp.parallel_layer, dict(heads=4, kv_heads=1, dim=64, vdim=64, chunk=33, rheads=2, rdim=64, rvdim=64)),
             (pp.parallel_layer, dict(ff=0, rheads=1, rdim=9, rvdim=11, heads=1, kv_heads=1, dim=5, vdim=3, chunk=7)),
             (pp.mamba2_layer, {}), (pp.mamba2_layer, dict(heads=4, vdim=64, state=64, groups=1, conv=4, norm_groups=4, ff=40)),
             (pp.mamba2_layer, dict(heads=2, vdim=3, state=5, groups=2, conv=1, norm_groups=1)),
             (pp.parallel2_layer, {}), (pp.parallel2_layer, dict(heads=8, kv_heads=2, dim=128, vdim=128, rot=64, scale=1.0, width=64, blocks=2, conv=4)),
             (pp.parallel2_layer, dict(ff=0, heads=3, kv_heads=1, dim=10, vdim=4, rot=10, width=21, blocks=3, conv=1))]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("make,over", ONE_LAYER)
def test_one_layer_whole_in_portions_and_token_by_token(gpu, dtype, make, over):
    cfg = pp.model([make(**over)])
    w = pp.random_weights(cfg, 51)
    toks = tokens(cfg, 110, 52)
    ref = pp.forward(cfg, w, toks)
    path = write_model(cfg, w)
    for cuts in ([110], [2, 70, 3, 2, 9, 16, 8], []):
        mostly(run_cut(path, dtype, toks, cuts), ref, dtype, f"{make.__name__} {over} cut {cuts[:3]}")


def one_branch(make, over, seed, branch):
    """A one-layer model of whose parallel members only one is heard: the other's norm weight is zero."""
    cfg = pp.model([make(ff=0, **over)])
    w = pp.random_weights(cfg, seed)
    w[f"l0.mix.{'right' if branch == 'left' else 'left'}.out"] *= 0.0
    return cfg, w


@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("dtype,page", [("float32", 8), ("bfloat16", 16)])
@pytest.mark.parametrize("over", [dict(chunk=24), dict(chunk=16, heads=4, kv_heads=1, dim=64, vdim=64), dict(chunk=65, dim=32, vdim=80), dict(chunk=1),
                                  dict(chunk=2), dict(chunk=32, heads=8, kv_heads=4, dim=64, vdim=128)])
def test_what_a_position_sees_begins_with_its_chunk(gpu, over, dtype, page, decoded):
    """At a chunk's first, second, a middle and its last place: the chunk's first token moves the logits as the plain
    implementation says, the token in front of the chunk not at all (the same bits), as a prompt and decoded."""
    C = over["chunk"]
    cfg, w = one_branch(pp.parallel_layer, over, 53, "left")
    path = write_model(cfg, w)
    base = tokens(cfg, 3 * C + 2, 54)
    for at in sorted({2 * C, min(2 * C + 1, 3 * C - 1), 2 * C + C // 2, 3 * C - 1}):
        toks, first = base[: at + 1], 2 * C
        cuts = ([at] if decoded else [at + 1])
        out = lambda t: run_cut(path, dtype, t, cuts, page=page)[-1]
        ref, got = pp.forward(cfg, w, toks)[-1], out(toks)
        mostly(got[None], ref[None], dtype, f"chunk {C} place {at}")
        other = list(toks)
        other[first] = (other[first] + 1) % cfg["vocab"]
        moved = pp.forward(cfg, w, other)[-1]
        got2 = out(other)
        mostly(got2[None], moved[None], dtype, f"chunk {C} place {at}: its first token changed")
        assert not np.array_equal(got, got2)
        for before in {first - 1, first - C, 0} - {first}:
            other = list(toks)
            other[before] = (other[before] + 1) % cfg["vocab"]
            assert np.array_equal(out(other), got), f"token {before} is outside the chunk of {at}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("over,page", [(dict(heads=4, kv_heads=2, dim=16, vdim=24, rot=8), 8), (dict(heads=4, kv_heads=1, dim=64, vdim=64, rot=32), 16),
                                       (dict(heads=4, kv_heads=2, dim=32, vdim=96, rot=0), 16)])
def test_a_far_key_that_stands_out(gpu, over, page, dtype):
    """Causal attention: a query that singles out one key hundreds of tokens back, at a page's first, last and middle place, in a
    prompt (short and long portions) and decoded alone.  What it brings is that key's value, so a wrong key would show."""
    cfg, w = one_branch(pp.parallel2_layer, dict(over, scale=0.5 if over["dim"] == 64 else 2.0), 65, "left")
    A, B = 7, 11
    w["l0.mix.left.out"] *= 4.0
    m = cfg["layers"][0]["mixer"]["left"]
    w["embed"][:, :2] = 0.0
    w["embed"][A, 0] = w["embed"][B, 1] = 8.0                     # the width's first coordinate is A's alone, its second B's
    d = m["dim"]
    for h in range(m["heads"]):
        w["l0.mix.left.q"][h * d + d - 1, 1] = 24.0                # an unrotated coordinate of every query head looks at B ...
    for c in range(m["kv_heads"]):
        w["l0.mix.left.k"][c * d + d - 1, :] = 0.0
        w["l0.mix.left.k"][c * d + d - 1, 0] = 24.0                # ... and meets the keys' that A alone lights up
    w = {k: torch.as_tensor(v).to(torch.bfloat16).double().numpy() for k, v in w.items()}
    path = write_model(cfg, w)
    for far in (0, page - 1, page, 5 * page + 3):
        toks = [t if t not in (A, B) else 20 for t in tokens(cfg, 420, 66)]
        toks[far], toks[-1] = A, B
        ref = pp.forward(cfg, w, toks)[-1]
        gone = list(toks)
        gone[far] = 20
        assert float(np.abs(ref - pp.forward(cfg, w, gone)[-1]).max()) > 0.5 * float(ref.std()), "the far key carries the answer"
        for cuts in ([420], [402], [419], [50, 300, 70]):
            mostly(run_cut(path, dtype, toks, cuts, page=page)[-1:], ref[None], dtype, f"key {far} cut {cuts}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("make,over", [(pp.mamba2_layer, {}), (pp.mamba2_layer, dict(heads=4, vdim=32, state=64, groups=2, conv=4)),
                                       (pp.parallel_layer, {}), (pp.parallel_layer, dict(rheads=2, rdim=64, rvdim=64)),
                                       (pp.parallel2_layer, {}), (pp.parallel2_layer, dict(width=64, blocks=2, conv=4))])
def test_a_far_token_through_the_state_alone(gpu, make, over, dtype):
    """Recurrences that forget almost nothing over 300 tokens (the attention beside them muted): the first token moves the last
    logits, whole, in portions and decoded, as the plain implementation says."""
    cfg, w = one_branch(make, over, 70, "right") if make is not pp.mamba2_layer else (pp.model([make(**over)]), None)
    if w is None:
        w = pp.random_weights(cfg, 70)
        w["l0.mix.A_log"] = w["l0.mix.A_log"] * 0 - 5.0
        w["l0.mix.dt_bias"] = w["l0.mix.dt_bias"] * 0 - 1.0
    elif make is pp.parallel_layer:
        w["l0.mix.right.f.b"] = w["l0.mix.right.f.b"] * 0 + 8.0
        w["l0.mix.right.i"][:, 0] = w["l0.mix.right.f"][:, 0] = 0.0
        w["l0.mix.right.i"][:, 0], w["embed"][:, 0], w["embed"][5, 0] = 2.0, 0.0, 4.0      # the first token opens the input gate
    else:
        w["l0.mix.right.lam"] = w["l0.mix.right.lam"] * 0 - 7.0
    w = {k: torch.as_tensor(v).to(torch.bfloat16).double().numpy() for k, v in w.items()}
    w["embed"][5] *= 16.0
    toks = [t if t != 5 else 6 for t in tokens(cfg, 300, 71)]
    other = [5] + toks[1:]
    path = write_model(cfg, w)
    ref, ref2 = pp.forward(cfg, w, toks)[-1], pp.forward(cfg, w, other)[-1]
    assert float(np.abs(ref - ref2).max()) > 3e-3 * float(ref.std()), "the plain logits at the end"
    for cuts in ([300], [2, 64, 65, 127, 40], [280]):
        a, b = run_cut(path, dtype, toks, cuts)[-1], run_cut(path, dtype, other, cuts)[-1]
        mostly(a[None], ref[None], dtype, f"cut {cuts}")
        mostly(b[None], ref2[None], dtype, f"cut {cuts}: another first token")


@pytest.mark.parametrize("dtype", DTYPES)
def test_gates_biases_and_norm_weights_show(gpu, dtype):
    """Output gates that all but close half the columns, branch norm weights that let one branch outweigh the other, biases of the
    recurrences and a convolution that reads the oldest tap alone."""
    toks = None
    for make, names in ((pp.parallel_layer, {"left.g": 8.0, "right.g": 8.0, "left.out": 5.0, "right.out": -4.0, "right.norm": 3.0, "right.i.b": 4.0, "right.f.b": -2.0}),
                        (pp.parallel2_layer, {"right.y.b": 3.0, "right.x.b": 3.0, "right.conv.b": 3.0, "right.ra.b": -4.0, "right.ri.b": 3.0, "left.out": 5.0}),
                        (pp.mamba2_layer, {"conv.b": 2.0, "dt_bias": 4.0, "D": -5.0, "norm": 3.0, "A_log": 2.0})):
        cfg = pp.model([make()])
        w = pp.random_weights(cfg, 75)
        toks = tokens(cfg, 40, 76)
        ref0 = pp.forward(cfg, w, toks)
        for name, size in names.items():
            v = w["l0.mix." + name]
            sign = np.where(np.arange(v.size).reshape(v.shape) % 2, 1.0, -0.25)
            w2 = dict(w, **{"l0.mix." + name: 8.0 * v if v.ndim == 2 and name.endswith(".g") else size * sign})
            ref = pp.forward(cfg, w2, toks)
            assert float(np.abs(ref - ref0).max()) > 0.1 * float(ref.std()), f"{name} matters"
            path = write_model(cfg, w2)
            mostly(run_cut(path, dtype, toks, [40]), ref, dtype, f"{name} whole")
            mostly(run_cut(path, dtype, toks, []), ref, dtype, f"{name} token by token")


# ---- whole models ----------------------------------------------------------------------------------------------------------
CONFIGS = {"s": (pp.tiny_config_s, 11, 8), "u": (pp.tiny_config_u, 12, 16), "w": (pp.tiny_config_w, 13, 4)}
NAMES = ["s", "u", "w"]


@functools.lru_cache(maxsize=None)
def folder(name):
    make, seed, _ = CONFIGS[name]
    cfg = make()
    w = pp.random_weights(cfg, seed)
    return write_model(cfg, w), cfg, w


@functools.lru_cache(maxsize=None)
def plain_logits(name, seed, length):
    _, cfg, w = folder(name)
    toks = tokens(cfg, length, 700 + seed)
    return toks, pp.forward(cfg, w, toks)


def runner(name, dtype, max_tokens, **kw):
    from prelude_amd.trace import TraceRunner
    return TraceRunner(folder(name)[0], dtype, max_tokens, page_size=CONFIGS[name][2], **kw)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompt_every_position(gpu, name, dtype):
    toks, ref = plain_logits(name, 0, 200)
    r = runner(name, dtype, 256, state_slots=2)
    got = r.step([{"id": "x", "tokens": toks, "want": list(range(len(toks)))}], ["x"])
    mostly(got, ref, dtype, f"{name} whole")
    assert r.engine.tables.audit() == "" and r.engine.tables.num_requests() == 0


@pytest.mark.parametrize("name", NAMES)
def test_every_layer_of_the_stream(gpu, name):
    """The stream after every layer, in 32-bit, against the plain one's."""
    from prelude_amd.ops import kernels as K
    toks, _ = plain_logits(name, 0, 200)
    _, cfg, w = folder(name)
    want = []
    pp.forward(cfg, w, toks[:60], streams=want)
    r = runner(name, "float32", 64, state_slots=1)
    seen = []
    for b in r.engine.model.blocks:
        def wrapped(*a, _f=b.forward, **k):
            h, res = _f(*a, **k)
            seen.append(res + K.as_tensor(h))      # the layer's output waits to be added
            return h, res
        b.forward = wrapped
    r.step([{"id": "x", "tokens": toks[:60], "want": [59]}], ["x"])
    assert len(seen) == len(want)
    for i, (a, b) in enumerate(zip(seen, want)):
        close(a, b, "float32", f"after layer {i}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_prefill_then_token_by_token(gpu, name, dtype):
    toks, ref = plain_logits(name, 1, 150)
    r = runner(name, dtype, 256, state_slots=1)
    n = 37                                  # a cut inside a page and inside every chunk
    outs = [r.step([{"id": 0, "tokens": toks[:n], "want": list(range(n))}])]
    for i in range(n, len(toks)):          # chunks begin and end among the decoded tokens; in bfloat16, replays of a captured step
        outs.append(r.step([{"id": 0, "tokens": [toks[i]], "want": [0]}]))
    mostly(np.concatenate(outs), ref, dtype, f"{name} decode")


def test_long_decoding_from_graphs_equals_steps_run_directly(gpu):
    """300 decoded tokens in bfloat16, replayed from captured steps, against the same steps run directly and against the plain
    logits."""
    toks, ref = plain_logits("u", 5, 330)
    runs = []
    for graphs in (True, False):
        r = runner("u", "bfloat16", 384, state_slots=1)
        if not graphs:
            r.engine._graphs = None
        outs = [r.step([{"id": 0, "tokens": toks[:30], "want": [29]}])]
        outs += [r.step([{"id": 0, "tokens": [t], "want": [0]}]) for t in toks[30:]]
        runs.append(np.concatenate(outs))
    mostly(runs[0], ref[29:], "bfloat16", "from graphs")
    # (the two differ where a step's class of contexts does: rounding only)
    assert float(np.abs(runs[0] - runs[1]).max()) <= 0.05 * float(np.std(ref))


def test_portions_replayed_from_graphs_equal_portions_run_directly(gpu):
    """The same portion sizes over and over, so that steps with portions are captured and replayed, with other requests' steps
    between the replays."""
    toks, ref = plain_logits("u", 6, 320)
    other, ref_other = plain_logits("u", 7, 90)
    r = runner("u", "bfloat16", 512, state_slots=2)
    outs, outs2, j = [], [], 0
    for i in range(0, 320, 20):
        outs.append(r.step([{"id": 0, "tokens": toks[i:i + 20], "want": list(range(20))}]))
        n = 1 if i % 40 else 8
        if j + n <= len(other):
            outs2.append(r.step([{"id": 1, "tokens": other[j: j + n], "want": list(range(n))}]))
            j += n
    mostly(np.concatenate(outs), ref, "bfloat16", "portions of one size")
    mostly(np.concatenate(outs2), ref_other[:j], "bfloat16", "another request between them")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_from_the_first_token_one_by_one(gpu, name, dtype):
    toks, ref = plain_logits(name, 2, 40)
    r = runner(name, dtype, 64, state_slots=1)
    outs = [r.step([{"id": 0, "tokens": [t], "want": [0]}]) for t in toks]
    mostly(np.concatenate(outs), ref, dtype, f"{name} one by one")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_portions_of_changing_size(gpu, name, dtype):
    toks, ref = plain_logits(name, 3, 330)
    sizes = [7, 2, 13, 2, 1, 31, 2, 9, 16, 3, 8, 2, 64, 5, 129, 2]
    r = runner(name, dtype, 512, state_slots=1)
    outs, i, k = [], 0, 0
    while i < len(toks):
        n = min(sizes[k % len(sizes)], len(toks) - i)
        k += 1
        outs.append(r.step([{"id": "p", "tokens": toks[i:i + n], "want": list(range(n))}]))
        i += n
    mostly(np.concatenate(outs), ref, dtype, f"{name} portions")


def test_the_32_bit_logits_do_not_depend_on_the_cut(gpu):
    toks, _ = plain_logits("s", 4, 90)
    runs = []
    for cuts in ([90], [1] * 90, [5, 2, 40, 1, 22, 20]):
        r = runner("s", "float32", 128, state_slots=1)
        outs, i = [], 0
        for c in cuts:
            outs.append(r.step([{"id": "c", "tokens": toks[i:i + c], "want": list(range(c))}]))
            i += c
        runs.append(np.concatenate(outs))
    for other in runs[1:]:
        assert float(np.abs(other - runs[0]).max()) <= 1e-5 * float(np.abs(runs[0]).max())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_unequal_requests_in_one_batch_with_pages_and_slots_used_again(gpu, name, dtype):
    """Six requests of unequal length through a pool that holds three of them and three state slots: portions of some
    beside single tokens of others; a request ends as soon as it is fed, and its pages and its slot go to the next."""
    lengths = [90, 17, 64, 33, 160, 5]
    seqs = [plain_logits(name, 10 + i, n) for i, n in enumerate(lengths)]
    r = runner(name, dtype, 3 * 192, state_slots=3)
    rng = np.random.default_rng(7)
    fed, waiting, live = [0] * len(seqs), list(range(len(seqs))), []
    got = [[] for _ in seqs]
    while waiting or live:
        while waiting and len(live) < 3:
            live.append(waiting.pop(0))
        entries, end = [], []
        for i in live:
            left = lengths[i] - fed[i]
            n = 1 if (fed[i] > 0 and rng.random() < 0.5) else int(min(left, rng.choice([2, 3, 16, 29, 40, 150])))
            entries.append({"id": f"r{i}", "tokens": seqs[i][0][fed[i]:fed[i] + n], "want": list(range(n))})
            fed[i] += n
            if fed[i] == lengths[i]:
                end.append(f"r{i}")
        out = r.step(entries, end)
        k = 0
        for e in entries:
            i = int(e["id"][1:])
            got[i].append(out[k:k + len(e["tokens"])])
            k += len(e["tokens"])
        live = [i for i in live if fed[i] < lengths[i]]
    for i, (toks, ref) in enumerate(seqs):
        mostly(np.concatenate(got[i]), ref, dtype, f"{name} request {i}")
    assert r.engine.tables.audit() == "" and r.engine.tables.num_requests() == 0
    assert r.engine.tables.free_state_slots() == 3


def test_a_batch_gives_what_each_request_gives_alone(gpu):
    """32-bit: a request's logits in a batch of unequal requests equal those it has alone, to rounding."""
    seqs = [plain_logits("s", 40 + i, n)[0] for i, n in enumerate([70, 9, 33])]
    alone = []
    for s in seqs:
        r = runner("s", "float32", 128, state_slots=1)
        alone.append(np.concatenate([r.step([{"id": 0, "tokens": s[:-4], "want": list(range(len(s) - 4))}])] +
                                    [r.step([{"id": 0, "tokens": [t], "want": [0]}]) for t in s[-4:]]))
    r = runner("s", "float32", 3 * 128, state_slots=3)
    first = r.step([{"id": i, "tokens": s[:-4], "want": list(range(len(s) - 4))} for i, s in enumerate(seqs)])
    tails = [r.step([{"id": i, "tokens": [s[len(s) - 4 + k]], "want": [0]} for i, s in enumerate(seqs)]) for k in range(4)]
    at = 0
    for i, s in enumerate(seqs):
        got = np.concatenate([first[at: at + len(s) - 4]] + [t[i:i + 1] for t in tails])
        at += len(s) - 4
        assert float(np.abs(got - alone[i]).max()) <= 1e-5 * float(np.abs(alone[i]).max()), f"request {i}"


def test_chunks_give_their_pages_back(gpu):
    """Attention inside chunks and recurrence alone: 600 tokens through a pool that holds little more than a chunk, then long
    decoding; a chunk's pages are free the moment the next one begins."""
    cfg = pp.model([pp.parallel_layer(heads=3, kv_heads=3, dim=12, vdim=20, chunk=40, rheads=1, rdim=5, rvdim=7, ff=12),
                    pp.mamba2_layer(heads=3, vdim=5, state=7, groups=1, conv=2, norm_groups=3)], width=36)
    w = pp.random_weights(cfg, 90)
    toks = tokens(cfg, 600, 91)
    from prelude_amd.trace import TraceRunner
    r = TraceRunner(write_model(cfg, w), "float32", 112, page_size=4, state_slots=1)
    outs, i = [], 0
    for n in [50, 3, 64] + [61] * 6 + [1] * 117:
        outs.append(r.step([{"id": "w", "tokens": toks[i:i + n], "want": list(range(n))}]))
        i += n
        assert r.engine.tables.live_pages(0, 0) <= -(-(n + 40) // 4) + 1
        if n == 1 and (i - 1) % 40 == 0:
            assert r.engine.tables.live_pages(0, 0) == 1, f"position {i - 1} begins a chunk"
    assert i == 600
    check(np.concatenate(outs), T(pp.forward(cfg, w, toks)), "float32", "a request longer than the pool")
    assert r.engine.tables.audit() == ""


def test_greedy_generation_through_the_scheduler(gpu):
    """``LLM.generate`` with temperature 0 gives the plain implementation's greedy tokens, for prompts of unequal length
    in one call (32-bit, so that no rounding decides between neighbours): the scheduler's portions, the token carried from
    one step to the next on the device, the slots."""
    from prelude_amd.llm import LLM
    path, cfg, w = folder("s")
    llm = LLM(path, dtype="float32", page_size=8, max_cache_tokens=512)
    prompts = [plain_logits("s", 30, 9)[0], plain_logits("s", 31, 31)[0], plain_logits("s", 32, 2)[0]]
    res = llm.generate(prompts, max_tokens=12, temperature=0.0)
    for p, out in zip(prompts, res):
        seq = list(p)
        for _ in range(12):
            seq.append(int(pp.forward(cfg, w, seq)[-1].argmax()))
        assert out.token_ids == seq[len(p):], f"prompt of {len(p)}"


def test_greedy_generation_in_bfloat16_from_graphs(gpu):
    """The same through the serving path (bfloat16, steps replayed from captured graphs, the next step launched before
    the last one's tokens are read): each generated token is the plain implementation's choice given the tokens before
    it, wherever that choice is not a close call."""
    from prelude_amd.llm import LLM
    path, cfg, w = folder("u")
    llm = LLM(path, dtype="bfloat16", page_size=16, max_cache_tokens=1024)
    prompts = [plain_logits("u", 33, 20)[0], plain_logits("u", 34, 3)[0]]
    res = llm.generate(prompts, max_tokens=24, temperature=0.0)
    clear = 0
    for p, out in zip(prompts, res):
        assert len(out.token_ids) == 24
        seq = list(p) + out.token_ids
        ref = pp.forward(cfg, w, seq)
        for k in range(24):
            row = ref[len(p) - 1 + k]
            top2 = np.sort(row)[-2:]
            if top2[1] - top2[0] > 0.3 * float(row.std()):
                clear += 1
                assert out.token_ids[k] == int(row.argmax()), f"prompt of {len(p)}, token {k}"
    assert clear >= 10


def test_command_line_with_the_pools_sized_from_free_memory(gpu, capsys):
    from prelude_amd import cli
    path, cfg, w = folder("u")
    prompt = tokens(cfg, 11, 740)
    assert cli.main(["--model", path, "--prompt-ids", ",".join(map(str, prompt)), "--max-tokens", "6", "--temperature", "0"]) == 0
    rec = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert rec["finish_reason"] == "length" and len(rec["token_ids"]) == 6
    ref = pp.forward(cfg, w, prompt)[-1]
    top2 = np.sort(ref)[-2:]
    if top2[1] - top2[0] > 0.25 * float(ref.std()):
        assert rec["token_ids"][0] == int(ref.argmax())
    assert cli.main(["--model", path, "--random-weights", "--prompt-len", "5", "--max-tokens", "3", "--max-cache-tokens", "256"]) == 0
    rec = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert len(rec["token_ids"]) == 3 and all(0 <= t < cfg["vocab"] for t in rec["token_ids"])


# ---- configurations drawn at random ------------------------------------------------------------------------------------
def draw_config(seed):
    """A Pogorax configuration drawn from a seed: any sizes the design allows, also ones no kernel is tuned for."""
    rng = np.random.default_rng(seed)
    pick = lambda xs: xs[int(rng.integers(0, len(xs)))]
    layers = []
    for _ in range(int(rng.integers(2, 6))):
        kind = pick(["mamba2", "parallel", "parallel_2"])
        ff = int(pick([0, 8, 24, 40, 64, 100]))
        if kind == "mamba2":
            groups, per = int(pick([1, 2, 3])), int(pick([1, 2, 4]))
            heads, vdim = groups * per, int(pick([4, 5, 8, 16, 24, 32, 64]))
            layers.append(pp.mamba2_layer(heads=heads, vdim=vdim, state=int(pick([4, 8, 16, 24, 33, 48, 64, 128])), groups=groups,
                                          conv=int(pick([1, 2, 3, 4, 4, 5])), norm_groups=int(pick([1, groups, heads])), ff=ff))
            continue
        kv, group = int(pick([1, 2, 3, 4])), int(pick([1, 2, 4]))
        dim = int(pick([6, 8, 16, 20, 32, 48, 64, 96]))
        vdim = int(pick([4, 8, 20, 24, 32, 64, 80, dim]))
        if kind == "parallel":
            layers.append(pp.parallel_layer(heads=kv * group, kv_heads=kv, dim=dim, vdim=vdim, scale=float(pick([0.5, 1.0, 2.0])) / math.sqrt(dim),
                                            chunk=int(pick([1, 2, 5, 16, 31, 32, 33, 64, 100])), rheads=int(pick([1, 2, 3, 5])),
                                            rdim=int(pick([4, 8, 16, 33, 64, 128])), rvdim=int(pick([4, 8, 24, 40, 70, 128])),
                                            cap=float(pick([3.0, 9.0, 15.0, 30.0])), ff=ff))
        else:
            blocks = int(pick([1, 2, 3, 5]))
            layers.append(pp.parallel2_layer(heads=kv * group, kv_heads=kv, dim=dim, vdim=vdim, scale=float(pick([0.1, 0.3, 1.0])),
                                             rot=int(pick([0, 2, dim // 2, dim])) // 2 * 2, base=float(pick([100.0, 1e4, 1e6])),
                                             width=blocks * int(pick([3, 8, 16, 24, 40, 72])), blocks=blocks, conv=int(pick([1, 2, 4, 4, 6])), ff=ff))
    cfg = pp.model(layers, width=int(pick([32, 36, 48, 64, 72, 96, 128, 160])), vocab=int(rng.integers(40, 400)),
                   scale=float(pick([1.0, 3.0, 8.0])), eps=float(pick([1e-6, 1e-5, 1e-4])))
    return cfg, int(pick([4, 8, 16, 32]))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("seed", list(range(int(os.environ.get("PRELUDE_AMD_DRAWN_CONFIGS", "12")))))   # widen for a hunt
def test_drawn_configuration(gpu, seed, dtype):
    """Each drawn model whole, then in portions beside a request that decodes, through a pool and state slots that are used again."""
    from prelude_amd.trace import TraceRunner
    cfg, page = draw_config(seed)
    toks = np.random.default_rng(2000 + seed).integers(0, cfg["vocab"], size=150).tolist()
    other = np.random.default_rng(3000 + seed).integers(0, cfg["vocab"], size=40).tolist()
    w = pp.random_weights(cfg, 300 + seed)
    ref, ref_other = pp.forward(cfg, w, toks), pp.forward(cfg, w, other)
    mv, mv_other = (pp.movement(cfg, w, t, seeds=3) for t in (toks, other)) if dtype == "bfloat16" else (None, None)
    at = lambda m, a, b: None if m is None else m[a:b]
    what = f"seed {seed} {dtype} page {page} {cfg}"
    r = TraceRunner(write_model(cfg, w), dtype, 256, page_size=page, state_slots=2)
    got = r.step([{"id": "w", "tokens": toks, "want": list(range(150))}], ["w"])
    mostly(got, ref, dtype, "whole: " + what, mv)
    a, b, i, j = [], [], 0, 10
    r.step([{"id": "o", "tokens": other[:10], "want": []}])
    for n in (3, 70, 2, 17, 1, 1, 40, 16):
        entries = [{"id": "p", "tokens": toks[i:i + n], "want": list(range(n))}]
        if j < len(other):
            entries.append({"id": "o", "tokens": [other[j]], "want": [0]})
        out = r.step(entries)
        a.append(out[:n])
        if j < len(other):
            b.append(out[n:])
            j += 1
        i += n
    mostly(np.concatenate(a), ref[:i], dtype, "portions: " + what, at(mv, 0, i))
    mostly(np.concatenate(b), ref_other[10:j], dtype, "decoding beside them: " + what, at(mv_other, 10, j))
    assert r.engine.tables.audit() == ""
