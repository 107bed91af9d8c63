"""Pogorax, plainly: one function per mechanism, in 64-bit, token by token where that is the clearest form.

Nothing here is shared with the product: no kernels, no parts, no cache.  A model is ``(cfg, w)``: the configuration as
the dictionary a config.json holds, and the tensors by name as float64 arrays.

The design.  x = embed[token] * scale.  A layer: x <- x + mixer(rms(x)), then, where it has a feed-forward,
x <- x + ff(rms(x)).  Mixers: ``mamba2`` (a state-space recurrence with one decay a token and head, behind a short
convolution); ``parallel`` (attention inside chunks of the sequence with a gate on its output, beside the matrix memory
of mLSTM) and ``parallel_2`` (causal attention on rotated unit queries and keys, beside Griffin's recurrent block), both
half the sum of their two members' outputs, each brought to unit RMS first.  Feed-forward: down(gelu(gate) * up), or none.
"""
import math

import numpy as np


def rms_unit(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def log_sigmoid(z):
    return np.minimum(z, 0.0) - np.log1p(np.exp(-np.abs(z)))


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rotate_pairs(x, positions, dims, base):
    """Turns the first ``dims`` dimensions of the last axis of x [T, heads, d], 2i with 2i + 1: the pair (u, v) at
    position p becomes (u cos a - v sin a, v cos a + u sin a), a = p * base^(-2i/dims)."""
    out = x.copy()
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        for t, p in enumerate(positions):
            c, s = math.cos(p * f), math.sin(p * f)
            u, v = x[t, :, 2 * i], x[t, :, 2 * i + 1]
            out[t, :, 2 * i] = u * c - v * s
            out[t, :, 2 * i + 1] = v * c + u * s
    return out


def visible(n, chunk=None):
    """[i, j]: whether the query at i sees the key at j: j <= i and, with ``chunk``, both in one chunk of that many places."""
    i = np.arange(n)
    see = i[:, None] >= i[None, :]
    return see & (i[:, None] // chunk == i[None, :] // chunk) if chunk else see


def softmax_sum(s, see, v):
    """One head's output from its scores s [T, T], what each query sees and its values v [T, dv]."""
    s = np.where(see, s, -np.inf)
    e = np.exp(s - s.max(axis=1, keepdims=True))
    return (e / e.sum(axis=1, keepdims=True)) @ v


def short_conv(x, w, b):
    """A causal convolution over time on each channel: x [T, C], w [C, taps], the last column the token's own."""
    taps = w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    return sum(padded[j: j + len(x)] * w[:, j] for j in range(taps)) + b


def attention(h, positions, w, m, eps):
    """Both attentions: rotation with norms behind it where the mixer has ``rot``, chunks where it has ``mask``, a gate on
    the output where there is a ``g``."""
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ w["q"].T).reshape(T, H, d)
    k = (h @ w["k"].T).reshape(T, G, d)
    v = (h @ w["v"].T).reshape(T, G, dv)
    if "rot" in m:
        q, k = (rms_unit(rotate_pairs(z, positions, m["rot"]["dims"], m["rot"]["base"]), eps) for z in (q, k))
    see = visible(T, m["mask"]["size"] if "mask" in m else None)
    o = np.stack([softmax_sum((q[:, a] @ k[:, a // (H // G)].T) * m["scale"], see, v[:, a // (H // G)]) for a in range(H)], axis=1)
    o = o.reshape(T, H * dv)
    if "g" in w:
        o = o * sigmoid(h @ w["g"].T)
    return o @ w["o"].T


def mlstm_recurrence(q, k, v, i, f, state=None):
    """q, k [T, heads, d], v [T, heads, dv], log gates i, f [T, heads] -> outputs [T, heads, dv] and (S, n, m) at the end."""
    T, H, d = q.shape
    S, n, m = (np.zeros((H, d, v.shape[2])), np.zeros((H, d)), np.zeros(H)) if state is None else (a.copy() for a in state)
    o = np.zeros_like(v)
    for t in range(T):
        new = np.maximum(f[t] + m, i[t])
        keep, add = np.exp(f[t] + m - new), np.exp(i[t] - new)
        S = keep[:, None, None] * S + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + add[:, None] * k[t]
        m = new
        den = np.maximum(np.abs((n * q[t]).sum(-1)), np.exp(-m)) + 1e-6
        o[t] = np.einsum("hde,hd->he", S, q[t]) / den[:, None]
    return o, (S, n, m)


def mlstm(h, w, m, eps):
    H, d, dv, cap = m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    T = h.shape[0]
    q = (h @ w["q"].T).reshape(T, H, d) * d ** -0.5
    k = (h @ w["k"].T).reshape(T, H, d)
    v = (h @ w["v"].T).reshape(T, H, dv)
    i = cap * np.tanh((h @ w["i"].T + w["i.b"]) / cap)
    f = log_sigmoid(cap * np.tanh((h @ w["f"].T + w["f.b"]) / cap))
    o, _ = mlstm_recurrence(q, k, v, i, f)
    o = rms_unit(o, eps).reshape(T, H * dv) * w["norm"] * sigmoid(h @ w["g"].T)
    return o @ w["o"].T


def ssd_recurrence(C, B, x, dt, A, D, state=None):
    """C, B [T, heads, N], x [T, heads, dv], steps dt [T, heads], rates A, skips D [heads]: S <- exp(-A dt) S + dt B x^T,
    y = S^T C + D x; outputs [T, heads, dv] and the state [heads, N, dv] at the end."""
    T, H, N = B.shape
    S = np.zeros((H, N, x.shape[2])) if state is None else state.copy()
    y = np.zeros_like(x)
    for t in range(T):
        S = np.exp(-A * dt[t])[:, None, None] * S + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        y[t] = np.einsum("hne,hn->he", S, C[t]) + D[:, None] * x[t]
    return y, S


def mamba2(h, w, m, eps):
    H, dv, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    T, inner = h.shape[0], H * dv
    p = h @ w["in"].T
    z, xbc, dt = p[:, :inner], p[:, inner: 2 * inner + 2 * G * N], p[:, 2 * inner + 2 * G * N:]
    xbc = silu(short_conv(xbc, w["conv"], w["conv.b"]))
    x = xbc[:, :inner].reshape(T, H, dv)
    B, C = (np.repeat(a.reshape(T, G, N), H // G, axis=1) for a in (xbc[:, inner: inner + G * N], xbc[:, inner + G * N:]))
    y, _ = ssd_recurrence(C, B, x, softplus(dt + w["dt_bias"]), np.exp(w["A_log"]), w["D"])
    y = y.reshape(T, inner) * silu(z)
    y = rms_unit(y.reshape(T, m["norm_groups"], -1), eps).reshape(T, inner) * w["norm"]
    return y @ w["o"].T


def lru_recurrence(u, r, i, lam, state=None):
    """u, r, i [T, width]: log a = -8 r softplus(lam), S <- a S + sqrt(1 - a^2) i u; S at every token, and at the end."""
    S = np.zeros(u.shape[1]) if state is None else state.copy()
    out = np.zeros_like(u)
    for t in range(len(u)):
        log_a = -8.0 * r[t] * softplus(lam)
        S = np.exp(log_a) * S + np.sqrt(-np.expm1(2.0 * log_a)) * i[t] * u[t]
        out[t] = S
    return out, S


def block_gate(u, w, b):
    """sigmoid(w[n] u_n + b[n]) for the equal parts u_n of u."""
    n, size, _ = w.shape
    parts = u.reshape(len(u), n, size)
    return sigmoid(np.stack([parts[:, a] @ w[a].T + b[a] for a in range(n)], axis=1)).reshape(u.shape)


def griffin(h, w, m):
    y = gelu_tanh(h @ w["y"].T + w["y.b"])
    u = short_conv(h @ w["x"].T + w["x.b"], w["conv"], w["conv.b"])
    S, _ = lru_recurrence(u, block_gate(u, w["ra"], w["ra.b"]), block_gate(u, w["ri"], w["ri.b"]), w["lam"])
    return (S * y) @ w["o"].T


def feed_forward(h, w):
    return (gelu_tanh(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def sub(w, prefix):
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def mixer(kind, h, positions, w, m, eps):
    if kind == "mamba2":
        return mamba2(h, w, m, eps)
    left, right = sub(w, "left."), sub(w, "right.")
    a = attention(h, positions, left, m["left"], eps)
    b = mlstm(h, right, m["right"], eps) if kind == "parallel" else griffin(h, right, m["right"])
    return 0.5 * (rms_unit(a, eps) * left["out"] + rms_unit(b, eps) * right["out"])


def layer(x, positions, cfg, w, i):
    lc, eps, p = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    x = x + mixer(lc["type"], rms_unit(x, eps) * w[p + "norm1"], positions, sub(w, p + "mix."), lc["mixer"], eps)
    if lc.get("mlp"):
        x = x + feed_forward(rms_unit(x, eps) * w[p + "norm2"], sub(w, p + "mlp."))
    return x


def forward(cfg, w, tokens, streams=None):
    """Logits [T, vocab] of a whole sequence; ``streams`` (a list) receives x after every layer."""
    x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    positions = list(range(len(tokens)))
    for i in range(len(cfg["layers"])):
        x = layer(x, positions, cfg, w, i)
        if streams is not None:
            streams.append(x.copy())
    return (rms_unit(x, cfg["norm"]["eps"]) * w["final.norm"]) @ w["head"].T


# ---- configurations and weights of the tests' own --------------------------------------------------------------------------
def _mlp(ff):
    return {"kind": "dense", "ff": ff} if ff else None


def mamba2_layer(heads=6, vdim=16, state=24, groups=3, conv=3, norm_groups=2, ff=0):
    return {"type": "mamba2", "mlp": _mlp(ff), "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                                         "norm_groups": norm_groups}}


def parallel_layer(heads=4, kv_heads=2, dim=16, vdim=24, chunk=20, scale=0.3, rheads=3, rdim=16, rvdim=24, cap=9.0, ff=40):
    return {"type": "parallel", "mlp": _mlp(ff),
            "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": chunk}},
                      "right": {"heads": rheads, "dim": rdim, "vdim": rvdim, "gate_cap": cap}}}


def parallel2_layer(heads=4, kv_heads=2, dim=16, vdim=24, rot=8, base=10000.0, scale=0.5, width=48, blocks=3, conv=5, ff=40):
    return {"type": "parallel_2", "mlp": _mlp(ff),
            "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"base": base, "dims": rot}},
                      "right": {"width": width, "blocks": blocks, "conv": conv}}}


def model(layers, width=48, vocab=90, scale=2.0, eps=1e-5):
    return {"architecture": "Pogorax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": layers}


def tiny_config_s():
    """Every mixer, with and without a feed-forward; heads over fewer KV heads; state groups of two heads."""
    return model([parallel_layer(), mamba2_layer(ff=32), parallel2_layer(), parallel_layer(heads=6, kv_heads=3, dim=8, vdim=8, chunk=33, ff=0),
                  mamba2_layer(heads=4, vdim=8, groups=1, norm_groups=4)])


def tiny_config_u():
    """Sizes the matrix cores take; one KV head; states larger than a chunk of tokens is long; a block for the whole width."""
    return model([parallel2_layer(heads=4, kv_heads=1, dim=64, vdim=64, rot=64, scale=0.2, width=64, blocks=1, conv=4),
                  mamba2_layer(heads=4, vdim=64, state=128, groups=4, conv=4, norm_groups=1),
                  parallel_layer(heads=4, kv_heads=1, dim=64, vdim=128, chunk=80, scale=0.125, rheads=2, rdim=64, rvdim=128, cap=20.0),
                  parallel_layer(heads=8, kv_heads=4, dim=32, vdim=32, chunk=65, scale=0.2, rheads=4, rdim=128, rvdim=32)],
                 width=64, vocab=120, scale=1.5)


def tiny_config_w():
    """As many KV heads as heads; chunks of one and two tokens; a convolution of one tap; odd sizes."""
    return model([parallel_layer(heads=3, kv_heads=3, dim=12, vdim=20, chunk=2, rheads=1, rdim=5, rvdim=7, cap=3.0, ff=12),
                  mamba2_layer(heads=3, vdim=5, state=7, groups=1, conv=1, norm_groups=3),
                  parallel2_layer(heads=1, kv_heads=1, dim=6, vdim=10, rot=2, width=15, blocks=5, conv=2, ff=0),
                  parallel_layer(heads=1, kv_heads=1, dim=4, vdim=4, chunk=1, rheads=5, rdim=20, rvdim=4, ff=20)],
                 width=36, vocab=50, scale=4.0, eps=1e-4)


def tensor_shapes(cfg):
    """Tensor name -> shape, as the design's files hold them."""
    h, v = cfg["width"], cfg["vocab"]
    t = {"embed": (v, h), "final.norm": (h,), "head": (v, h)}
    for i, lc in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lc["mixer"]
        t[p + "norm1"] = (h,)
        if lc.get("mlp"):
            ff = lc["mlp"]["ff"]
            t.update({p + "norm2": (h,), p + "mlp.gate": (ff, h), p + "mlp.up": (ff, h), p + "mlp.down": (h, ff)})
        p += "mix."
        if lc["type"] == "mamba2":
            H, inner, gn = m["heads"], m["heads"] * m["vdim"], m["groups"] * m["state"]
            t.update({p + "in": (2 * inner + 2 * gn + H, h), p + "conv": (inner + 2 * gn, m["conv"]), p + "conv.b": (inner + 2 * gn,),
                      p + "dt_bias": (H,), p + "A_log": (H,), p + "D": (H,), p + "norm": (inner,), p + "o": (h, inner)})
            continue
        a, b = m["left"], m["right"]
        l, r = p + "left.", p + "right."
        t.update({l + "q": (a["heads"] * a["dim"], h), l + "k": (a["kv_heads"] * a["dim"], h), l + "v": (a["kv_heads"] * a["vdim"], h),
                  l + "o": (h, a["heads"] * a["vdim"]), l + "out": (h,), r + "out": (h,)})
        if lc["type"] == "parallel":
            H, d, dv = b["heads"], b["dim"], b["vdim"]
            t.update({l + "g": (a["heads"] * a["vdim"], h), r + "q": (H * d, h), r + "k": (H * d, h), r + "v": (H * dv, h),
                      r + "g": (H * dv, h), r + "o": (h, H * dv), r + "norm": (H * dv,), r + "i": (H, h), r + "i.b": (H,),
                      r + "f": (H, h), r + "f.b": (H,)})
        else:
            n, k = b["width"], b["blocks"]
            t.update({r + "y": (n, h), r + "y.b": (n,), r + "x": (n, h), r + "x.b": (n,), r + "conv": (n, b["conv"]), r + "conv.b": (n,),
                      r + "ra": (k, n // k, n // k), r + "ra.b": (k, n // k), r + "ri": (k, n // k, n // k), r + "ri.b": (k, n // k),
                      r + "lam": (n,), r + "o": (h, n)})
    return t


def random_weights(cfg, seed):
    """Weights that bfloat16 holds exactly, as float64 arrays: matrices N(0, 1/sqrt(inputs)), norm weights around 1,
    biases, decays and gates of a size that shows: memories of a few tokens beside memories of hundreds."""
    import torch
    g = torch.Generator().manual_seed(seed)
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        n = torch.randn(shape, generator=g)
        if last in ("norm1", "norm2", "norm", "out"):
            x = 1.0 + 0.2 * n
        elif name.endswith(".f.b"):
            x = 3.0 + n
        elif last == "dt_bias":
            x = n - 2.0
        elif last == "A_log":
            x = 0.7 * n
        elif last == "D":
            x = 1.0 + 0.3 * n
        elif last == "lam":
            x = n - 3.0
        elif last == "b":
            x = 0.3 * n
        elif last == "conv":
            x = n / math.sqrt(shape[-1])
        elif last == "embed":
            x = n
        else:
            x = n / math.sqrt(shape[-1])
        w[name] = x.to(torch.bfloat16).to(torch.float64).numpy()
    return w


def movement(cfg, w, toks, seeds=2, size=2.0 ** -9):
    """How far every position's logits move, in units of their spread, when every weight is off by a random part of its last
    bfloat16 place: the largest over a few draws.  What rounding to bfloat16 does to a model is of this size."""
    ref = forward(cfg, w, toks)
    out = np.zeros(len(toks))
    for s in range(seeds):
        g = np.random.default_rng(s)
        moved = forward(cfg, {k: v * (1.0 + size * g.standard_normal(v.shape)) for k, v in w.items()}, toks)
        out = np.maximum(out, np.abs(moved - ref).max(axis=1) / ref.std())
    return out
