"""Pugavik on the GPU against the plain implementation (``plain_pugavik``): every mechanism's kernels alone and as a
one-layer model, then the engine under schedules (whole, token by token, portions down to two tokens, unequal requests in
one batch, pages and state slots used again, long decoding) and greedy generation through ``LLM`` and the command line.
Configurations and weights are the tests' own; where random weights would hide a fault (a key at a window's edge or far
away, a sink, the heads' mixing, a decay near 0 or 1), inputs are made so that it shows."""
import functools
import json
import math
import os
import tempfile
import types

import numpy as np
import pytest
import torch

import plain_pugavik as pp
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


def mostly(got, ref, dtype, what):
    """Every row against the plain logits: 32-bit to rounding; bfloat16 to a quarter of the spread everywhere and to a
    tenth at nine rows in ten (the tests' models are narrow)."""
    ref = T(ref)
    if dtype == "float32":
        return check(got, ref, dtype, what)
    got = torch.as_tensor(got).double().reshape(ref.shape)
    err = (got - ref).abs().reshape(len(ref), -1).max(dim=1).values / float(ref.std())
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


# ---- norm, stream, embedding, activation --------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden", [36, 37, 48, 320, 2056, 5000, 9000])
def test_layer_norm_with_what_waits_added(gpu, dtype, hidden):
    """Rows with a mean far from zero (the variance is that of the deviations); what waits as a tensor, as slices, absent;
    chosen rows of the sum with the stream left alone."""
    from prelude_amd.ops import kernels as K
    n = 5
    x = torch.randn((n, hidden), generator=torch.Generator().manual_seed(1)) * 2 + torch.tensor([0.0, 30.0, -7.0, 100.0, 1.0])[:, None]
    w, b = 1 + 0.3 * torch.randn(hidden, generator=torch.Generator().manual_seed(2)), torch.randn(hidden, generator=torch.Generator().manual_seed(3))
    y = rnd((n, hidden), 4, dtype)
    parts = torch.randn((3, n, hidden), generator=torch.Generator().manual_seed(5))
    norm = lambda s: pp.layer_norm(s.double().numpy(), w.double().numpy(), b.double().numpy(), 1e-5)
    wd, bd = w.to(gpu), b.to(gpu)
    bound = lambda got, want, what: close(got, want, dtype, what)
    s = x.clone().to(gpu)
    bound(K.layer_norm_step(None, s, wd, bd, 1e-5, TD[dtype]), norm(x), "nothing waits")
    assert torch.equal(s.cpu(), x)
    s = x.clone().to(gpu)
    bound(K.layer_norm_step(y.to(gpu), s, wd, bd, 1e-5, TD[dtype]), norm(x + y.float()), "a tensor waits")
    close(s, x.double() + y.double(), "float32", "the stream took it", scale=100.0)
    s = x.clone().to(gpu)
    sl = K.SliceSums(parts.to(gpu), TD[dtype])
    bound(K.layer_norm_step(sl, s, wd, bd, 1e-5, TD[dtype]), norm((x.double() + parts.double().sum(0)).float()), "slices wait")
    s = x.clone().to(gpu)
    rows = torch.tensor([3, 0, 3], dtype=torch.int32, device=gpu)
    for what, want in ((y.to(gpu), x + y.float()), (sl, (x.double() + parts.double().sum(0)).float()), (None, x)):
        bound(K.layer_norm_step(what, s, wd, bd, 1e-5, TD[dtype], rows=rows), norm(want)[[3, 0, 3]], "chosen rows")
        assert torch.equal(s.cpu(), x), "read only"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden", [37, 64])
def test_stream_sums_scaled_embedding_and_activation(gpu, dtype, hidden):
    from prelude_amd.ops import kernels as K
    n = 6
    g = lambda s: torch.randn((n, hidden), generator=torch.Generator().manual_seed(s))
    x, extra, row, y = g(1) * 20, g(2), torch.randn(hidden, generator=torch.Generator().manual_seed(3)), rnd((n, hidden), 4, dtype)
    dev = lambda t: None if t is None else t.to(gpu)
    for yy, ee, rr in ((y, extra, row), (None, extra, None), (y, None, None), (None, None, row), (None, None, None)):
        s = x.clone().to(gpu)
        out = K.stream_sum(s, dev(yy), dev(ee), dev(rr))
        want = x.double() + sum(t.double() for t in (yy, ee, rr) if t is not None)
        close(out, want, "float32", "a fresh sum")
        assert torch.equal(s.cpu(), x)
        assert K.stream_sum(s, dev(yy), dev(ee), dev(rr), out=s) is s
        close(s, want, "float32", "in place")
    table, ids = rnd((50, hidden), 5, dtype), torch.tensor([3, 49, 0, 3], dtype=torch.int32)
    got = K.embed_scaled(ids.to(gpu), table.to(gpu), 3.5)
    assert got.dtype == torch.float32
    close(got, table.double()[[3, 49, 0, 3]] * 3.5, "float32", "rows times a number")
    wide = rnd((n, hidden * 3 + 8), 6, dtype, scale=4.0)
    wide[0, hidden + 8], wide[1, hidden + 9], wide[2, hidden + 10] = 60.0, -60.0, 0.0
    out = torch.full((n, hidden * 2 + 16), 9.0, dtype=TD[dtype], device=gpu)
    K.activate(wide.to(gpu)[:, hidden + 8: 2 * hidden + 8], "gelu_tanh", out[:, 8: hidden + 8], 0.5)
    close(out[:, 8: hidden + 8], 0.5 * pp.gelu_tanh(wide[:, hidden + 8: 2 * hidden + 8].double().numpy()), "float32" if dtype == "float32" else dtype,
          "columns of wider rows", scale=8.0 if dtype == "bfloat16" else 30.0)
    assert (out[:, :8] == 9.0).all() and (out[:, hidden + 8:] == 9.0).all(), "nothing beside them"


# ---- queries, keys and values in front of the mixed scores ----------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nh,nkv,hd,vd,rot,bias,norm,vnorm,page", [
    (4, 2, 16, 24, 8, True, True, True, 8), (6, 3, 8, 8, 8, True, True, True, 4), (3, 3, 12, 20, 0, True, True, True, 8),
    (4, 1, 64, 32, 64, False, True, False, 16), (8, 4, 130, 200, 100, True, False, True, 16), (1, 1, 5, 7, 2, False, False, False, 8),
    (16, 4, 64, 128, 64, True, True, True, 16)])
def test_prepare_in_front_of_mixed_scores(gpu, dtype, nh, nkv, hd, vd, rot, bias, norm, vnorm, page):
    from prelude_amd.ops import kernels as K
    n, base, off, eps = 21, 777.0, 5, 1e-5
    nq, nk, nv = nh * hd, nkv * hd, nkv * vd
    p = rnd((n, off + nq + nk + nv + 3), 11, dtype)
    g = torch.Generator().manual_seed(12)
    biases = tuple(0.5 * torch.randn(s, generator=g) for s in (nq, nk, nv)) if bias else None
    qw, kw = (1 + 0.3 * torch.randn(hd, generator=g) for _ in range(2)) if norm else (None, None)
    talk = torch.randn((nh, nh), generator=g)
    freq = torch.tensor([base ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=torch.float64).float() if rot else None
    pos = list(range(100, 100 + n))
    x = p.double().numpy()[:, off:]
    parts = [x[:, :nq], x[:, nq: nq + nk], x[:, nq + nk: nq + nk + nv]]
    if bias:
        parts = [a + b.double().numpy() for a, b in zip(parts, biases)]
    q, k, v = parts[0].reshape(n, nh, hd), parts[1].reshape(n, nkv, hd), parts[2].reshape(n, nkv, vd)
    if norm:
        q, k = pp.rms_unit(q, eps) * qw.double().numpy(), pp.rms_unit(k, eps) * kw.double().numpy()
    if rot:
        q, k = pp.rotate_pairs(q, pos, rot, base), pp.rotate_pairs(k, pos, rot, base)
    if vnorm:
        v = pp.rms_unit(v, eps)
    mixed = np.zeros((n, nh, nkv, hd))
    tk = talk.double().numpy()
    for a in range(nh):
        mixed[:, :, a // (nh // nkv)] += tk[None, :, a, None] * q[:, None, a]
    pages = -(-n // page) + 2
    perm = torch.randperm(pages, generator=g).tolist()
    slots = torch.tensor([perm[i // page] * page + i % page for i in range(n)], dtype=torch.int32, device=gpu)
    kc = torch.full((pages, 1, page, nk), 7.0, dtype=TD[dtype], device=gpu)
    vc = torch.full((pages, nkv, vd, page), 7.0, dtype=TD[dtype], device=gpu)
    dev = lambda t: None if t is None else t.to(gpu)
    out = K.talking_prepare(p.to(gpu), off, off + nq, off + nq + nk, None if biases is None else tuple(dev(b) for b in biases), dev(qw), dev(kw),
                            dev(freq), torch.tensor(pos, dtype=torch.int32, device=gpu), dev(talk), slots, kc, vc, nh, nkv, hd, vd, rot,
                            vnorm, eps)
    close(out, mixed.reshape(n, nh, nk), dtype, "mixed queries", scale=float(np.abs(mixed).max()))
    kc, vc = kc.cpu(), vc.cpu()
    ks = torch.cat([kc[perm[j], 0] for j in range(-(-n // page))])[:n]
    vs = torch.cat([vc[perm[j]].permute(2, 0, 1) for j in range(-(-n // page))])[:n]
    close(ks, k.reshape(n, nk), dtype, "keys side by side", scale=float(np.abs(k).max()))
    close(vs, v, dtype, "values", scale=float(np.abs(v).max()))
    assert (kc[perm[-1]] == 7.0).all() and (vc[perm[-1]] == 7.0).all(), "another page is left alone"


# ---- attention on the matrix cores for any widths ---------------------------------------------------------------------------
WIDE = [  # heads, key heads, value heads, key width, value width, window, page
    (4, 1, 2, 112, 88, 60, 16), (4, 1, 2, 32, 24, 24, 8), (16, 1, 4, 256, 128, 200, 16), (20, 1, 5, 40, 12, 0, 16), (3, 1, 3, 136, 64, 1, 8),
    (4, 4, 4, 192, 128, 0, 16), (6, 3, 3, 48, 36, 65, 32), (4, 4, 2, 64, 128, 130, 16), (2, 1, 1, 512, 256, 0, 16), (2, 1, 2, 264, 100, 33, 64),
    (5, 1, 1, 8, 4, 0, 8), (8, 1, 8, 128, 200, 128, 16), (34, 1, 2, 64, 64, 0, 16)]


@pytest.mark.parametrize("nh,nk,nv,kd,vd,window,page", WIDE)
def test_attention_for_any_widths(gpu, nh, nk, nv, kd, vd, window, page):
    """Portions (a whole prompt over several tiles, one behind a prefix, two tokens) beside single tokens at contexts of one
    key, one block and many, through shuffled pages whose other places hold large numbers; for every query head one far key, and
    the key just inside and just outside the window, are made to stand out."""
    from prelude_amd.ops import kernels as K
    assert K.attention_wide_supported(kd, vd, page)
    ctx = [300, 140, 70, 1, 128, 561, 9]
    qn = [300, 33, 2, 1, 1, 1, 1]
    step = step_of(ctx, qn, gpu, page=page)
    g = torch.Generator().manual_seed(20)
    scale = kd ** -0.5
    sink = torch.randn(nh, generator=g)
    need = [-(-c // page) for c in ctx]
    perm = torch.randperm(sum(need) + 2, generator=g).tolist()
    kc = torch.full((len(perm), nk, page, kd), 30.0, dtype=torch.bfloat16)
    vc = torch.full((len(perm), nv, vd, page), -30.0, dtype=torch.bfloat16)
    table = torch.full((len(ctx), max(need)), perm[-1], dtype=torch.int32)
    qs, wants, at = [], [], 0
    for s, (c, n) in enumerate(zip(ctx, qn)):
        k, v = torch.randn((c, nk, kd), generator=g), torch.randn((c, nv, vd), generator=g).to(torch.bfloat16)
        q = torch.randn((n, nh, kd), generator=g).to(torch.bfloat16)
        last = q[-1].float()
        for key in {0, c // 3, c - window, c - window - 1} if window else {0, c // 3}:
            if 0 <= key < c:
                for a in range(nk):
                    k[key, a] = 6.0 * last[a * (nh // nk)] / last[a * (nh // nk)].norm() / scale ** 0.5
        k = k.to(torch.bfloat16)
        for j in range(need[s]):
            pg = perm[at]
            at += 1
            # pages wholly before every query's window have been given back
            if window and (j + 1) * page <= c - n - window + 1:
                table[s, j] = -1
                continue
            table[s, j] = pg
            m = min(page, c - j * page)
            kc[pg, :, :m] = k[j * page: j * page + m].transpose(0, 1)
            vc[pg, :, :, :m] = v[j * page: j * page + m].permute(1, 2, 0)
        qs.append(q)
        see = pp.visible(c, window or None)[c - n:]
        kk, vv, qq = k.double().numpy(), v.double().numpy(), q.double().numpy()
        o = np.zeros((n, nh, vd))
        for a in range(nh):
            kv = a // (nh // nk)
            o[:, a] = pp.softmax_sum(qq[:, a] @ kk[:, kv].T * scale, see, vv[:, kv % nv if nv <= nk else a // (nh // nv)], float(sink[a]))
        wants.append(o.reshape(n, nh * vd))
    group = types.SimpleNamespace(block_table=table.to(gpu))
    wide = torch.full((sum(qn), nh * vd + 12), 5.0, dtype=torch.bfloat16, device=gpu)
    q = torch.cat(qs).to(gpu)
    got = K.attention_wide(q, kc.to(gpu), vc.to(gpu), group, step, window, scale, sink=sink.to(gpu), out=wide[:, 4: 4 + nh * vd])
    want = np.concatenate(wants)
    close(got, want, "bfloat16", "attention", scale=max(1.0, float(np.abs(want).max())))
    assert (wide[:, :4] == 5.0).all() and (wide[:, 4 + nh * vd:] == 5.0).all(), "nothing beside the heads"
    alone = K.attention_wide(q, kc.to(gpu), vc.to(gpu), group, step, window, scale, sink=sink.to(gpu))
    assert torch.equal(alone, got.contiguous())
    # the kernel on the vector units, which the 32-bit engine and other widths use, says the same
    plain = K.attention_masked(q, kc.to(gpu), vc.to(gpu), group, step, window, 0, scale, sink=sink.to(gpu)) if kd <= 512 else None
    close(plain, want, "bfloat16", "attention on the vector units", scale=max(1.0, float(np.abs(want).max())))


@pytest.mark.parametrize("n,ctx", [(1, 5000), (3, 2600), (40, 700)])
def test_splits_of_a_single_tokens_context(gpu, n, ctx):
    """Many splits, and the same step cut otherwise: a far key that stands out, contexts that end inside a split."""
    from prelude_amd.ops import kernels as K
    nh, nv, kd, vd, page = 4, 2, 64, 32, 16
    lens = [ctx - 7 * i for i in range(n)]
    step = step_of(lens, [1] * n, gpu, page=page)
    g = torch.Generator().manual_seed(22)
    need = -(-ctx // page)
    kc = torch.randn((n * need, 1, page, kd), generator=g).to(torch.bfloat16)
    vc = torch.randn((n * need, nv, vd, page), generator=g).to(torch.bfloat16)
    table = torch.randperm(n * need, generator=g).to(torch.int32).reshape(n, need)
    q = torch.randn((n, nh, kd), generator=g).to(torch.bfloat16)
    scale = kd ** -0.5
    for s in range(n):
        far = lens[s] // 4
        kc[table[s, far // page], 0, far % page] = (9.0 * q[s, 0].float() / q[s, 0].float().norm() / scale ** 0.5).to(torch.bfloat16)
    want = []
    for s in range(n):
        k = kc[table[s].long(), 0].reshape(-1, kd)[: lens[s]].double().numpy()
        v = vc[table[s].long()].permute(0, 3, 1, 2).reshape(-1, nv, vd)[: lens[s]].double().numpy()
        o = [pp.softmax_sum(q[s, a:a + 1].double().numpy() @ k.T * scale, np.ones((1, lens[s]), bool), v[:, a // 2]) for a in range(nh)]
        want.append(np.concatenate(o, axis=1)[0])
    group = types.SimpleNamespace(block_table=table.to(gpu))
    args = (q.to(gpu), kc.to(gpu), vc.to(gpu), group, step, 0, scale)
    close(K.attention_wide(*args), np.stack(want), "bfloat16", "as planned")
    plan = K.SHARED_SPLIT_KEYS
    try:
        for keys in (256, 1024, 8192):
            K.SHARED_SPLIT_KEYS = (keys,)
            close(K.attention_wide(*args), np.stack(want), "bfloat16", f"splits of {keys}")
    finally:
        K.SHARED_SPLIT_KEYS = plan


# ---- gated linear attention ------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,d,e,rank,tau", [(3, 16, 24, 8, 8.0), (2, 64, 64, 16, 1.0), (1, 5, 7, 3, 3.0), (4, 128, 130, 16, 16.0), (2, 40, 100, 5, 0.5)])
def test_gated_linear_attention_across_cuts(gpu, dtype, heads, d, e, rank, tau):
    """Three sequences in portions (long ones in chunks in bfloat16, token by token in 32-bit), single tokens beside them, a
    slot left alone; channels that forget everything at once and channels that forget nothing."""
    from prelude_amd.ops import kernels as K
    g = torch.Generator().manual_seed(30)
    a2 = (torch.randn((heads * d, rank), generator=g) / rank ** 0.5).to(TD[dtype])
    bias = 2 + torch.randn(heads * d, generator=g)
    bias[:: 7], bias[1:: 7] = 60.0, -60.0 * tau       # sigmoid's ends: a decay of 1 and one of e^-60
    off, qk, vv = 8, heads * d, heads * e
    width = off + 2 * qk + vv + rank + 4
    lens = [333, 6, 150]
    seqs = [rnd((n, width), 31 + n, dtype) for n in lens]
    want, ends = [], []
    for s in seqs:
        x = s.double().numpy()[:, off:]
        z = x[:, 2 * qk + vv: 2 * qk + vv + rank] @ a2.double().numpy().T + bias.double().numpy()
        alpha = (pp.sigmoid(z) ** (1.0 / tau)).reshape(-1, heads, d)
        o, S = pp.gla_recurrence(x[:, :qk].reshape(-1, heads, d) * d ** -0.5, x[:, qk: 2 * qk].reshape(-1, heads, d),
                                 x[:, 2 * qk: 2 * qk + vv].reshape(-1, heads, e), alpha)
        want.append(o)
        ends.append(S)
    state = torch.full((5, heads, d, e), 3.0, device=gpu)
    slots = [3, 0, 4]
    state[slots] = 0.0
    cuts = [[1, 1, 200, 2, 65, 64], [2, 1, 1, 2], [130, 7, 1, 12]]
    got, fed = [[] for _ in seqs], [0, 0, 0]
    for k in range(6):
        live = [i for i in range(3) if k < len(cuts[i])]
        qn = [cuts[i][k] for i in live]
        p = torch.cat([seqs[i][fed[i]: fed[i] + cuts[i][k]] for i in live]).to(gpu)
        st = step_of([fed[i] + cuts[i][k] for i in live], qn, gpu, slots=[slots[i] for i in live])
        out = K.gated_linear_attention(p, off, off + qk, off + 2 * qk, off + 2 * qk + vv, a2.to(gpu), bias.to(gpu), tau, state, st, heads, d, e)
        at = 0
        for i, n in zip(live, qn):
            got[i].append(out[at: at + n].cpu())
            at += n
            fed[i] += n
    assert fed == lens
    # inputs are what they are in both formats and everything behind them is 32-bit: the bound is 32-bit's, loosened for the
    # hardware's exponential behind bfloat16 projections
    tol = 1.0 if dtype == "float32" else 4.0
    for i in range(3):
        close(torch.cat(got[i]), want[i], "float32", f"sequence {i}", scale=tol * float(np.abs(want[i]).max()))
        close(state[slots[i]], ends[i], "float32", f"the state of sequence {i}", scale=tol * float(np.abs(ends[i]).max()))
    assert (state[[1, 2]] == 3.0).all(), "another request's slot is left alone"


def test_recurrence_in_32_bit_does_not_depend_on_the_cut(gpu):
    from prelude_amd.ops import kernels as K
    heads, d, e, rank, n = 2, 32, 48, 4, 140
    g = torch.Generator().manual_seed(33)
    a2, bias = torch.randn((heads * d, rank), generator=g).to(gpu), (2 + torch.randn(heads * d, generator=g)).to(gpu)
    p = torch.randn((n, 2 * heads * d + heads * e + rank), generator=g).to(gpu)
    cols = (0, heads * d, 2 * heads * d, 2 * heads * d + heads * e)
    runs = []
    for cuts in ([140], [1] * 140, [70, 2, 1, 67]):
        state = torch.zeros((1, heads, d, e), device=gpu)
        outs, i = [], 0
        for c in cuts:
            outs.append(K.gated_linear_attention(p[i:i + c].contiguous(), *cols, a2, bias, 4.0, state, step_of([i + c], [c], gpu), heads, d, e))
            i += c
        runs.append((torch.cat(outs), state))
    for o, s in runs[1:]:
        assert float((o - runs[0][0]).abs().max()) <= 2e-6 * float(runs[0][0].abs().max())
        assert float((s - runs[0][1]).abs().max()) <= 2e-6 * float(runs[0][1].abs().max())


# ---- latents expanded into every head's keys and values ---------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,d,v,rank,rot,page", [(3, 16, 24, 40, 8, 8), (2, 128, 128, 64, 64, 16), (1, 5, 7, 12, 2, 8), (4, 32, 64, 24, 0, 32)])
def test_expanded_keys_values_and_queries(gpu, dtype, heads, d, v, rank, rot, page):
    from prelude_amd.ops import kernels as K
    g = torch.Generator().manual_seed(40)
    ctx = [page * 2 + 5, 3, page]
    table = torch.randperm(sum(-(-c // page) for c in ctx), generator=g).to(torch.int32)
    bt, at = torch.zeros((3, 3), dtype=torch.int32), 0
    for s, c in enumerate(ctx):
        m = -(-c // page)
        bt[s, :m] = table[at: at + m]
        at += m
    cache = rnd((at, page, rank + rot), 41, dtype)
    seq = torch.cat([torch.full((c,), s, dtype=torch.int32) for s, c in enumerate(ctx)])
    pos = torch.cat([torch.arange(c, dtype=torch.int32) for c in ctx])
    first = [0, -(-ctx[0] // page), -(-ctx[0] // page) + 1]
    slots = torch.cat([torch.arange(c, dtype=torch.int32) + first[s] * page for s, c in enumerate(ctx)])
    kv = rnd((sum(ctx), heads * (d + v)), 42, dtype)
    k_out = torch.full((first[2] + 2, heads, page, d + rot), 2.0, dtype=TD[dtype], device=gpu)
    v_out = torch.full((first[2] + 2, heads, v, page), 2.0, dtype=TD[dtype], device=gpu)
    dev = lambda t: t.to(gpu)
    K.latent_expand(dev(kv), dev(cache), dev(bt), dev(seq), dev(pos), dev(slots), k_out, v_out, heads, d, v, rank)
    k_out, v_out = k_out.cpu(), v_out.cpu()
    for i in range(sum(ctx)):
        pg, o = divmod(int(slots[i]), page)
        tail = cache[bt[seq[i], int(pos[i]) // page], int(pos[i]) % page, rank:]
        assert torch.equal(k_out[pg, :, o, :d].reshape(-1), kv[i, : heads * d]) and (k_out[pg, :, o, d:] == tail).all()
        assert torch.equal(v_out[pg, :, :, o].reshape(-1), kv[i, heads * d:])
    assert (k_out[-1] == 2.0).all() and (v_out[-1] == 2.0).all()
    wide = rnd((9, heads * (d + rot) + 16), 43, dtype)
    q = wide[:, 8: 8 + heads * (d + rot)].unflatten(1, (heads, d + rot))
    freq = torch.tensor([500.0 ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=torch.float64).float() if rot else None
    got = K.latent_queries(wide.to(gpu)[:, 8: 8 + heads * (d + rot)].unflatten(1, (heads, d + rot)), None if freq is None else dev(freq),
                           torch.arange(50, 59, dtype=torch.int32, device=gpu), d, rot)
    want = q.double().numpy().copy()
    if rot:
        want[:, :, d:] = pp.rotate_pairs(want[:, :, d:], range(50, 59), rot, 500.0)
    close(got, want, dtype, "queries")
    assert torch.equal(got[:, :, :d].cpu(), q[:, :, :d])


# ---- one-layer models ----------------------------------------------------------------------------------------------------
def write_model(cfg, w):
    from prelude_amd.weights import write_safetensors
    tmp = tempfile.TemporaryDirectory(prefix="prelude_amd_pugavik_")
    _keep.append(tmp)
    with open(os.path.join(tmp.name, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(tmp.name, "model.safetensors"), {k: torch.as_tensor(v).to(torch.bfloat16) for k, v in w.items()})
    return tmp.name


def run_cut(path, dtype, toks, cuts, page=8, max_tokens=512):
    """The logits of every position with the sequence fed in portions of ``cuts`` (the rest one by one)."""
    from prelude_amd.trace import TraceRunner
    r = TraceRunner(path, dtype, max_tokens, page_size=page, state_slots=1)
    outs, i, k = [], 0, 0
    while i < len(toks):
        n = min(cuts[k], len(toks) - i) if k < len(cuts) else 1
        k += 1
        outs.append(r.step([{"id": "s", "tokens": toks[i:i + n], "want": list(range(n))}]))
        i += n
    return np.concatenate(outs)


def tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


ONE_LAYER = [(pp.attention_layer, {}), (pp.attention_layer, dict(heads=3, kv_heads=3, dim=20, vdim=12, rot=0, window=7)),
             (pp.attention_layer, dict(heads=4, kv_heads=1, dim=64, vdim=128, rot=64, window=70, scale=0.125)),
             (pp.attention_layer, dict(heads=1, kv_heads=1, dim=6, vdim=10, rot=6, window=1, ff=0)),
             (pp.attention_layer, dict(heads=6, kv_heads=2, dim=100, vdim=72, rot=50, window=33, scale=0.1)),
             (pp.gla_layer, {}), (pp.gla_layer, dict(heads=2, dim=64, vdim=64, tau=1.0, ff=0)), (pp.gla_layer, dict(heads=1, dim=130, vdim=70, tau=20.0)),
             (pp.latent_layer, {}), (pp.latent_layer, dict(heads=4, dim=32, rot_dim=32, vdim=32, kv_rank=64)),
             (pp.latent_layer, dict(heads=2, dim=20, rot_dim=2, vdim=40, kv_rank=13, ff=0))]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("make,over", ONE_LAYER)
def test_one_layer_whole_in_portions_and_token_by_token(gpu, dtype, make, over):
    cfg = pp.model([make(**over)], loop=(0, 1, 2))
    w = pp.random_weights(cfg, 50)
    toks = tokens(cfg, 130, 51)
    ref = pp.forward(cfg, w, toks)
    path = write_model(cfg, w)
    for cuts in ([130], [60], [7, 2, 13, 2, 1, 31, 2, 9, 16, 3, 8, 2, 30], []):
        mostly(run_cut(path, dtype, toks if cuts else toks[:60], cuts), ref if cuts else ref[:60], dtype, f"{make.__name__} {over} cut {cuts[:3]}")


@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("dtype,page", [("float32", 8), ("bfloat16", 16)])
@pytest.mark.parametrize("over", [dict(window=24), dict(window=16, heads=4, kv_heads=1, dim=64, vdim=64, rot=32), dict(window=65, dim=32, vdim=80),
                                  dict(window=1), dict(window=2, heads=2, kv_heads=2)])
def test_what_a_position_sees_ends_at_the_edge_of_its_window(gpu, over, dtype, page, decoded):
    """A one-layer model: another token one place outside the window leaves the last logits bit for bit as they are (also on the
    matrix cores); at the window's oldest key it moves them as in the plain implementation.  For the last position of a
    prompt, and for a token decoded alone behind a prompt cut in the middle of a page."""
    window = over["window"]
    cfg = pp.model([pp.attention_layer(**over)])
    w = pp.random_weights(cfg, 60)
    path = write_model(cfg, w)
    n = 2 * window + 81
    toks = tokens(cfg, n, 61)
    cuts = [n - 19] if decoded else [n]

    def last(t):
        return run_cut(path, dtype, t, cuts, page=page)[-1]

    def other(c):
        t = list(toks)
        t[c] = (t[c] + 1 + c) % cfg["vocab"]
        return t
    base, ref = last(toks), pp.forward(cfg, w, toks)
    oldest = n - window
    for c in (oldest - 1, oldest - 2):
        assert np.array_equal(last(other(c)), base), f"token {c} is outside what {n - 1} sees"
    want = pp.forward(cfg, w, other(oldest))[-1]
    moved, got = want - ref[-1], last(other(oldest)) - base
    assert float(np.abs(moved).max()) > 1e-4 * float(ref.std()), "the plain logits move"
    if dtype == "float32":
        check(last(other(oldest)), T(want), dtype, f"token {oldest} is inside what {n - 1} sees")
    else:
        size = float(np.abs(moved).max())
        assert float(np.abs(got).max()) > 0 and float(np.abs(got - moved).max()) <= 0.5 * size + 0.04 * float(ref.std()), \
            f"token {oldest} is inside what {n - 1} sees"


def standing_out(make, over, seed):
    """A one-layer model in which the queries of token B's positions single out token A's keys far back: the width's first
    coordinate is A's alone and its second B's, keys and queries meet there with a score no other pair has."""
    cfg = pp.model([make(ff=0, **over)], width=48)
    w = pp.random_weights(cfg, seed)
    A, B = 7, 11
    m = cfg["layers"][0]["mixer"]
    w["embed"][:, :2] = 0.0
    w["embed"][A, 0] = w["embed"][B, 1] = 8.0
    H, d = m["heads"], m["dim"]
    for h in range(H):
        row = h * (d + m["rot_dim"])
        w["l0.mix.q"][row, 1] = 24.0                    # an unrotated query coordinate of every head looks at B ...
        w["l0.mix.uk"][h * d, :] = 0.0
        w["l0.mix.uk"][h * d, 0] = 4.0                  # ... and meets the latent's first coordinate, which A lights up
    w["l0.mix.dkv"][0, 0] = 24.0
    return cfg, {k: torch.as_tensor(v).to(torch.bfloat16).double().numpy() for k, v in w.items()}, A, B


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("over,page", [(dict(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=40), 8), (dict(heads=4, dim=32, rot_dim=32, vdim=32, kv_rank=64), 16)])
def test_a_far_key_that_stands_out(gpu, over, page, dtype):
    """Attention through latents without a window: a query that singles out one key hundreds of tokens back, at a page's
    first, last and middle place, in a prompt (short and long portions) and decoded alone.  What it brings is that key's
    value, so a wrong key, place or position would show."""
    cfg, w, A, B = standing_out(pp.latent_layer, over, 65)
    path = write_model(cfg, w)
    for far in (0, page - 1, page, 5 * page + 3):
        toks = [t if t not in (A, B) else 20 for t in tokens(cfg, 420, 66)]
        toks[far], toks[-1] = A, B
        ref = pp.forward(cfg, w, toks)[-1]
        gone = list(toks)
        gone[far] = 20
        assert float(np.abs(ref - pp.forward(cfg, w, gone)[-1]).max()) > 0.5 * float(ref.std()), "the far key carries the answer"
        for cuts in ([420], [402], [419], [50, 300, 70]):
            got = run_cut(path, dtype, toks, cuts, page=page)[-1:]
            if dtype == "float32":      # scores of several hundred: their own rounding moves the weights
                assert float(np.abs(got[0] - ref).max()) <= 5e-4 * float(np.abs(ref).max()), f"key {far} cut {cuts}"
            else:
                assert float(np.abs(got[0] - ref).max()) <= 0.25 * float(ref.std()), f"key {far} cut {cuts}"


@pytest.mark.parametrize("over,page", [(dict(heads=2, dim=64, rot_dim=32, vdim=64, kv_rank=64), 16), (dict(heads=3, dim=16, rot_dim=8, vdim=64, kv_rank=40), 8),
                                       (dict(heads=1, dim=128, rot_dim=64, vdim=128, kv_rank=96), 16)])
def test_long_portions_attend_through_expanded_latents(gpu, over, page, monkeypatch):
    """Under the bfloat16 engine a long portion has every head's keys and values made from the latents it can see, in
    temporary pages, where short ones and single tokens attend to the latents themselves: whole, behind a prefix that ends
    inside a page, beside a sequence that decodes, and the same prompt with the expanded form switched off."""
    from prelude_amd.parts.latent_attention import LatentAttention
    from prelude_amd.trace import TraceRunner
    cfg = pp.model([pp.latent_layer(**over)], loop=(0, 1, 2), width=64)
    w = pp.random_weights(cfg, 80)
    toks, other = tokens(cfg, 700, 81), tokens(cfg, 60, 82)
    ref, ref_other = pp.forward(cfg, w, toks), pp.forward(cfg, w, other)
    path = write_model(cfg, w)
    used = []
    real = LatentAttention._expanded
    monkeypatch.setattr(LatentAttention, "_expanded", lambda self, *a: used.append(1) or real(self, *a))
    monkeypatch.setattr(LatentAttention, "EXPAND_FROM_TOKENS", 100)
    r = TraceRunner(path, "bfloat16", 1024, page_size=page, state_slots=2)
    mostly(r.step([{"id": "w", "tokens": toks, "want": list(range(700))}], ["w"]), ref, "bfloat16", "whole")
    assert len(used) == 2, "both runs of the layer expanded"
    outs = [r.step([{"id": "p", "tokens": toks[:53], "want": list(range(53))}])]
    assert len(used) == 2, "a short portion attends to the latents themselves"
    r.step([{"id": "o", "tokens": other[:40], "want": []}])
    outs.append(r.step([{"id": "p", "tokens": toks[53:400], "want": list(range(347))}]))
    both = r.step([{"id": "p", "tokens": toks[400:], "want": list(range(300))}, {"id": "o", "tokens": [other[40]], "want": [0]}])
    assert len(used) == 6
    mostly(np.concatenate(outs + [both[:300]]), ref, "bfloat16", "portions behind a prefix")
    mostly(both[300:], ref_other[40:41], "bfloat16", "a single token beside a long portion")
    monkeypatch.setattr(LatentAttention, "EXPAND_FROM_TOKENS", 1 << 30)
    r2 = TraceRunner(path, "bfloat16", 1024, page_size=page, state_slots=1)
    mostly(r2.step([{"id": "w", "tokens": toks, "want": list(range(700))}], ["w"]), ref, "bfloat16", "without the expanded form")
    assert len(used) == 6


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_sink_a_mixing_matrix_and_biases_show(gpu, dtype):
    """Sinks far above the scores in every other head (those heads all but vanish, also at the first token, where a softmax
    without a sink gives the only key the weight 1), a mixing matrix that is no symmetric one and swaps heads, and large biases."""
    cfg = pp.model([pp.attention_layer(heads=4, kv_heads=2, dim=16, vdim=24, window=24)])
    w = pp.random_weights(cfg, 70)
    toks = tokens(cfg, 40, 71)
    ref0 = pp.forward(cfg, w, toks)
    base = {"l0.mix.sink": np.array([6.0, -3.0, 6.0, -3.0]),
            "l0.mix.talk": np.array([[0.0, 0.0, 2.0, 0.0], [0.0, 0.0, 0.0, 1.0], [0.0, 1.0, 0.0, 0.0], [-1.5, 0.0, 0.0, 0.25]]),
            "l0.mix.q.b": 2.0 * np.ones(64), "l0.mix.k.b": np.tile([1.5, -1.5], 16), "l0.mix.v.b": np.tile([2.0, -1.0], 24)}
    for name, value in base.items():
        w2 = dict(w, **{name: value})
        ref = pp.forward(cfg, w2, toks)
        assert float(np.abs(ref - ref0).max()) > 0.3 * float(ref.std()), f"{name} matters"
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
def test_every_run_of_the_stream(gpu, name):
    """The stream after every run of a layer (a looped layer counts each time), in 32-bit, against the plain one's."""
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
    assert len(seen) == len(want) == len(pp.run_order(cfg))
    for i, (a, b) in enumerate(zip(seen, want)):
        close(a, b, "float32", f"after run {i}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_prefill_then_token_by_token(gpu, name, dtype):
    toks, ref = plain_logits(name, 1, 150)
    r = runner(name, dtype, 256, state_slots=1)
    n = 37                                  # a cut inside a page and inside every window
    outs = [r.step([{"id": 0, "tokens": toks[:n], "want": list(range(n))}])]
    for i in range(n, len(toks)):          # every window passes over decoded tokens; in bfloat16, replays of a captured step
        outs.append(r.step([{"id": 0, "tokens": [toks[i]], "want": [0]}]))
    mostly(np.concatenate(outs), ref, dtype, f"{name} decode")


def test_long_decoding_from_graphs_equals_steps_run_directly(gpu):
    """300 decoded tokens in bfloat16, replayed from captured steps, against the same steps run directly (the same bits) and
    against the plain logits."""
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


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_token_far_back_moves_the_last_logits(gpu, dtype):
    """The recurrence and the attention without a window carry a token hundreds of places; the engine follows the plain
    implementation with it and without it."""
    toks, ref = plain_logits("s", 20, 260)
    _, cfg, w = folder("s")
    for c in (259 - 200, 0):
        other = list(toks)
        other[c] = (toks[c] + 1) % cfg["vocab"]
        ref2 = pp.forward(cfg, w, other)
        assert float(np.abs(ref[-1] - ref2[-1]).max()) > 1e-3 * float(ref.std()), f"the plain logits at the end, token {c}"
        r = runner("s", dtype, 640, state_slots=2)
        assert r.step([{"id": "a", "tokens": toks[:129], "want": []}]) is None
        a = r.step([{"id": "a", "tokens": toks[129:], "want": [130]}], ["a"])
        b = r.step([{"id": "b", "tokens": other, "want": [259]}], ["b"])
        mostly(a, ref[-1:], dtype, "as it is")
        mostly(b, ref2[-1:], dtype, f"with token {c} changed")


def test_windows_give_their_pages_back(gpu):
    """Windowed attention and recurrence alone: 600 tokens through a pool of 192, then long decoding."""
    cfg = pp.model([pp.attention_layer(heads=3, kv_heads=3, dim=12, vdim=20, rot=4, window=40), pp.gla_layer(heads=1, dim=5, vdim=7, tau=3.0)], width=36)
    w = pp.random_weights(cfg, 90)
    toks = tokens(cfg, 600, 91)
    from prelude_amd.trace import TraceRunner
    r = TraceRunner(write_model(cfg, w), "float32", 192, page_size=4, state_slots=1)
    outs, i = [], 0
    for n in [50, 3, 64] + [61] * 6 + [1] * 117:
        outs.append(r.step([{"id": "w", "tokens": toks[i:i + n], "want": list(range(n))}]))
        i += n
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
    cfg = pp.tiny_config_u()
    for lc in cfg["layers"]:
        if lc["type"] == "gla":
            lc["mixer"]["rank"] = 32     # drawn weights need a size where the file would have given it
    w = pp.random_weights(cfg, 12)
    path = write_model(cfg, w)
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
    """A Pugavik configuration drawn from a seed: any sizes the design allows, also ones no kernel is tuned for."""
    rng = np.random.default_rng(seed)
    pick = lambda xs: xs[int(rng.integers(0, len(xs)))]
    layers = []
    for _ in range(int(rng.integers(2, 6))):
        kind = pick(["attention", "gla", "latent_attention"])
        ff = int(pick([0, 8, 24, 40, 64, 100]))
        kv, group = int(pick([1, 2, 3, 4])), int(pick([1, 2, 4]))
        scale = lambda dim: float(pick([0.5, 1.0, 2.0])) / math.sqrt(dim)
        if kind == "attention":
            dim = int(pick([5, 8, 16, 20, 32, 48, 64]))
            layers.append(pp.attention_layer(heads=kv * group, kv_heads=kv, dim=dim, vdim=int(pick([4, 8, 20, 24, 32, 64, 80])),
                                             window=int(pick([1, 2, 5, 16, 31, 32, 33, 64, 100])), rot=int(pick([0, 2, dim // 2, dim])) // 2 * 2,
                                             base=float(pick([100.0, 1e4, 1e6])), scale=scale(dim), ff=ff))
        elif kind == "gla":
            layers.append(pp.gla_layer(heads=kv, dim=int(pick([4, 8, 16, 33, 64])), vdim=int(pick([4, 8, 24, 40, 70])),
                                       tau=float(pick([1.0, 4.0, 16.0])), ff=ff))
        else:
            dim = int(pick([4, 8, 16, 32, 64]))
            layers.append(pp.latent_layer(heads=kv * group, dim=dim, rot_dim=int(pick([2, 8, 16, 32])), vdim=int(pick([8, 16, 24, 64])),
                                          kv_rank=int(pick([8, 12, 16, 40, 64, 96])), base=float(pick([100.0, 1e4])), scale=scale(dim), ff=ff))
    n = len(layers)
    loop = None
    if rng.random() < 0.8:
        start = int(rng.integers(0, n + 1))
        loop = (start, int(rng.integers(start, n + 1)), int(pick([1, 2, 3])))
    cfg = pp.model(layers, width=int(pick([32, 36, 48, 64, 72, 96, 128, 160])), vocab=int(rng.integers(40, 400)), loop=loop,
                   scale=float(pick([1.0, 3.0, 8.0])), eps=float(pick([1e-6, 1e-5, 1e-4])))
    return cfg, int(pick([4, 8, 16, 32]))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("seed", list(range(int(os.environ.get("PRELUDE_AMD_DRAWN_CONFIGS", "12")))))   # widen for a hunt
def test_drawn_configuration(gpu, seed, dtype, monkeypatch):
    """Each drawn model whole, then in portions beside a request that decodes, through a pool and state slots that are
    used again; portions of 64 tokens or more attend through expanded latents where the drawn head sizes allow it."""
    from prelude_amd.parts.latent_attention import LatentAttention
    from prelude_amd.trace import TraceRunner
    monkeypatch.setattr(LatentAttention, "EXPAND_FROM_TOKENS", 64)
    cfg, page = draw_config(seed)
    toks = np.random.default_rng(2000 + seed).integers(0, cfg["vocab"], size=150).tolist()
    other = np.random.default_rng(3000 + seed).integers(0, cfg["vocab"], size=40).tolist()
    w = pp.random_weights(cfg, 300 + seed)
    ref, ref_other = pp.forward(cfg, w, toks), pp.forward(cfg, w, other)
    what = f"seed {seed} {dtype} page {page} {cfg}"
    r = TraceRunner(write_model(cfg, w), dtype, 256, page_size=page, state_slots=2)
    got = r.step([{"id": "w", "tokens": toks, "want": list(range(150))}], ["w"])
    mostly(got, ref, dtype, "whole: " + what)
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
    mostly(np.concatenate(a), ref[:i], dtype, "portions: " + what)
    mostly(np.concatenate(b), ref_other[10:j], dtype, "decoding beside them: " + what)
    assert r.engine.tables.audit() == ""
