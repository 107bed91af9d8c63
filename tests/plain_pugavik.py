"""Pugavik, plainly: one function per mechanism, in 64-bit, token by token where that is the clearest form.

Nothing here is shared with the product: no kernels, no parts, no cache.  A model is ``(cfg, w)``: the configuration as
the dictionary a config.json holds, and the tensors by name as float64 arrays.

The design.  x = embed[token] * scale.  Layers ``loop.start .. loop.stop - 1`` run ``loop.times`` times in a row with the
same weights; in front of pass t the embedding is added to x once more (not in front of pass 0) and then the row
``loop.step[t]``.  A layer: h = layernorm(x), x <- x + (mixer(h) + ff(h)), one norm for both.  Mixers: grouped-query
attention under a window with biases, queries and keys normed per head and rotated in pairs, values over their own root
mean square, the heads' scores mixed by a matrix, a sink; gated linear attention (a decay per key channel and token);
attention through a latent with a shared rotated key part.  Feed-forward: down(gelu(up)), or none.
"""
import math

import numpy as np


def rms_unit(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def layer_norm(x, w, b, eps):
    c = x - np.mean(x, axis=-1, keepdims=True)
    return c / np.sqrt(np.mean(c * c, axis=-1, keepdims=True) + eps) * w + b


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-np.clip(z, -700.0, 700.0)))


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


def mix_scores(s, talk):
    """score_h <- sum_g talk[h, g] score_g; s [heads, ...]."""
    return np.tensordot(talk, s, axes=(1, 0))


def visible(n, window=None):
    """[i, j]: whether the query at i sees the key at j: j <= i, and i - j < window."""
    d = np.arange(n)[:, None] - np.arange(n)[None, :]
    return (d >= 0) & (d < (window if window else n))


def softmax_sum(s, see, v, sink=None):
    """One head's output from its scores s [T, T], what each query sees, its values v [T, dv] and a number whose
    exponential is one more term of the denominator."""
    s = np.where(see, s, -np.inf)
    m = s.max(axis=1, keepdims=True)
    if sink is not None:
        m = np.maximum(m, sink)
    e = np.exp(s - m)
    den = e.sum(axis=1, keepdims=True)
    if sink is not None:
        den = den + np.exp(sink - m)
    return (e / den) @ v


def windowed_attention(h, positions, w, m, eps):
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ w["q"].T + w["q.b"]).reshape(T, H, d)
    k = (h @ w["k"].T + w["k.b"]).reshape(T, G, d)
    v = (h @ w["v"].T + w["v.b"]).reshape(T, G, dv)
    q, k = rms_unit(q, eps) * w["q.norm"], rms_unit(k, eps) * w["k.norm"]
    rot = m.get("rot")
    if rot and rot["dims"]:
        q, k = rotate_pairs(q, positions, rot["dims"], rot["base"]), rotate_pairs(k, positions, rot["dims"], rot["base"])
    v = rms_unit(v, eps)
    s = np.stack([(q[:, a] @ k[:, a // (H // G)].T) * m["scale"] for a in range(H)])
    s = mix_scores(s, w["talk"])
    see = visible(T, m["mask"]["size"])
    o = np.stack([softmax_sum(s[a], see, v[:, a // (H // G)], w["sink"][a]) for a in range(H)], axis=1)
    return o.reshape(T, H * dv) @ w["o"].T


def gla_recurrence(q, k, v, alpha, state=None):
    """q, k, alpha [T, heads, d], v [T, heads, dv] -> outputs [T, heads, dv] and the state [heads, d, dv] at the end:
    S <- diag(alpha) S + k v^T, o = S^T q."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2])) if state is None else state.copy()
    o = np.zeros_like(v)
    for t in range(T):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hde,hd->he", S, q[t])
    return o, S


def gated_linear_attention(h, w, m, eps):
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ w["q"].T).reshape(T, H, d) * d ** -0.5
    k = (h @ w["k"].T).reshape(T, H, d)
    v = (h @ w["v"].T).reshape(T, H, dv)
    z = ((h @ w["a1"].T) @ w["a2"].T + w["a2.b"]).reshape(T, H, d)
    alpha = sigmoid(z) ** (1.0 / m["tau"])
    o, _ = gla_recurrence(q, k, v, alpha)
    o = (rms_unit(o, eps) * w["norm"]).reshape(T, H * dv)
    return (o * silu(h @ w["g"].T)) @ w["o"].T


def latent_attention(h, positions, w, m, eps):
    H, d, r, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    T = h.shape[0]
    q = (h @ w["q"].T).reshape(T, H, d + r)
    down = h @ w["dkv"].T
    c = rms_unit(down[:, :rank], eps) * w["dkv.norm"]
    kr, qr = down[:, None, rank:], q[:, :, d:]
    if r:
        kr, qr = rotate_pairs(kr, positions, r, m["rot"]["base"]), rotate_pairs(qr, positions, r, m["rot"]["base"])
    k = (c @ w["uk"].T).reshape(T, H, d)
    v = (c @ w["uv"].T).reshape(T, H, dv)
    see = visible(T)
    o = np.stack([softmax_sum((q[:, a, :d] @ k[:, a].T + qr[:, a] @ kr[:, 0].T) * m["scale"], see, v[:, a]) for a in range(H)], axis=1)
    return o.reshape(T, H * dv) @ w["o"].T


def feed_forward(h, w):
    return gelu_tanh(h @ w["up"].T) @ w["down"].T


def sub(w, prefix):
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def layer(x, positions, cfg, w, i):
    lc, eps = cfg["layers"][i], cfg["norm"]["eps"]
    p = f"l{i}."
    h = layer_norm(x, w[p + "norm1"], w[p + "norm1.b"], eps)
    mw, m = sub(w, p + "mix."), lc["mixer"]
    if lc["type"] == "attention":
        y = windowed_attention(h, positions, mw, m, eps)
    elif lc["type"] == "gla":
        y = gated_linear_attention(h, mw, m, eps)
    elif lc["type"] == "latent_attention":
        y = latent_attention(h, positions, mw, m, eps)
    else:
        raise ValueError(lc["type"])
    if lc.get("mlp"):
        y = y + feed_forward(h, sub(w, p + "mlp."))
    return x + y


def run_order(cfg):
    """(layer, pass) in the order they run; pass is None outside the loop."""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        out += [(i, t) for i in range(loop["start"], loop["stop"])]
    return out + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg, w, tokens, streams=None):
    """Logits [T, vocab] of a whole sequence; ``streams`` (a list) receives x after every layer run."""
    e = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    x = e
    positions = list(range(len(tokens)))
    loop = cfg.get("loop")
    for i, t in run_order(cfg):
        if t is not None and i == loop["start"]:
            if t > 0:
                x = x + e
            x = x + w["loop.step"][t]
        x = layer(x, positions, cfg, w, i)
        if streams is not None:
            streams.append(x.copy())
    return layer_norm(x, w["final.norm"], w["final.norm.b"], cfg["norm"]["eps"]) @ w["head"].T


# ---- configurations and weights of the tests' own --------------------------------------------------------------------------
def attention_layer(heads=4, kv_heads=2, dim=16, vdim=24, window=24, rot=8, base=10000.0, scale=0.3, ff=40):
    return {"type": "attention", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": window},
                      "rot": {"base": base, "dims": rot}}}


def gla_layer(heads=3, dim=16, vdim=24, tau=8.0, ff=40):
    return {"type": "gla", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}}


def latent_layer(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=40, base=5000.0, scale=0.25, ff=40):
    return {"type": "latent_attention", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                      "rot": {"base": base, "dims": rot_dim}}}


def model(layers, width=48, vocab=90, loop=None, scale=2.0, eps=1e-5):
    cfg = {"architecture": "Pugavik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "layers": layers}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def tiny_config_s():
    """Every mixer once, the two in the middle run three times; heads over fewer KV heads; a layer without a feed-forward."""
    return model([attention_layer(), gla_layer(), latent_layer(ff=0), attention_layer(heads=6, kv_heads=3, dim=8, vdim=8, rot=8,
                                                                                      window=40)], loop=(1, 3, 3))


def tiny_config_u():
    """The whole model run twice; sizes the matrix cores take; one KV head; values wider and narrower than the keys."""
    return model([latent_layer(heads=4, dim=32, rot_dim=32, vdim=32, kv_rank=64), gla_layer(heads=2, dim=64, vdim=64, tau=1.0),
                  attention_layer(heads=4, kv_heads=1, dim=64, vdim=32, rot=64, window=70, scale=0.125),
                  attention_layer(heads=8, kv_heads=4, dim=32, vdim=64, rot=16, window=33, scale=0.2)],
                 width=64, vocab=120, loop=(0, 4, 2), scale=1.5)


def tiny_config_w():
    """No loop; as many KV heads as heads; windows of one and two keys; nothing rotated in the attention; odd sizes."""
    return model([attention_layer(heads=3, kv_heads=3, dim=12, vdim=20, rot=0, window=2, ff=12), gla_layer(heads=1, dim=5, vdim=7, tau=3.0, ff=20),
                  latent_layer(heads=1, dim=4, rot_dim=2, vdim=12, kv_rank=12, ff=0), attention_layer(heads=1, kv_heads=1, dim=6, vdim=6, rot=2,
                                                                                               window=1, ff=16)],
                 width=36, vocab=50, scale=4.0, eps=1e-4)


def tensor_shapes(cfg):
    """Tensor name -> shape, as the design's files hold them."""
    h, v = cfg["width"], cfg["vocab"]
    t = {"embed": (v, h), "final.norm": (h,), "final.norm.b": (h,), "head": (v, h)}
    if cfg.get("loop"):
        t["loop.step"] = (cfg["loop"]["times"], h)
    for i, lc in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lc["mixer"]
        t[p + "norm1"], t[p + "norm1.b"] = (h,), (h,)
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        if lc["type"] == "attention":
            G = m["kv_heads"]
            for n, rows in (("q", H * d), ("k", G * d), ("v", G * dv)):
                t[f"{p}mix.{n}"], t[f"{p}mix.{n}.b"] = (rows, h), (rows,)
            t.update({p + "mix.q.norm": (d,), p + "mix.k.norm": (d,), p + "mix.talk": (H, H), p + "mix.sink": (H,)})
        elif lc["type"] == "gla":
            r = m.get("rank", max(2, d // 2))
            t.update({p + "mix.q": (H * d, h), p + "mix.k": (H * d, h), p + "mix.v": (H * dv, h), p + "mix.g": (H * dv, h),
                      p + "mix.norm": (dv,), p + "mix.a1": (r, h), p + "mix.a2": (H * d, r), p + "mix.a2.b": (H * d,)})
        else:
            r, rank = m["rot_dim"], m["kv_rank"]
            t.update({p + "mix.q": (H * (d + r), h), p + "mix.dkv": (rank + r, h), p + "mix.dkv.norm": (rank,),
                      p + "mix.uk": (H * d, rank), p + "mix.uv": (H * dv, rank)})
        t[p + "mix.o"] = (h, H * dv)
        if lc.get("mlp"):
            ff = lc["mlp"]["ff"]
            t[p + "mlp.up"], t[p + "mlp.down"] = (ff, h), (h, ff)
    return t


def random_weights(cfg, seed):
    """Weights that bfloat16 holds exactly, as float64 arrays: matrices N(0, 1/sqrt(inputs)), norm weights around 1,
    biases, sinks, the heads' mixing and the loop's vectors of a size that shows."""
    import torch
    g = torch.Generator().manual_seed(seed)
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm"):
            x = 1.0 + 0.2 * torch.randn(shape, generator=g)
        elif name.endswith("a2.b"):
            x = 2.0 + torch.randn(shape, generator=g)
        elif last == "b":
            x = 0.3 * torch.randn(shape, generator=g)
        elif last == "sink":
            x = 0.7 * torch.randn(shape, generator=g)
        elif last == "talk":
            x = torch.eye(shape[0]) + 0.3 * torch.randn(shape, generator=g)
        elif name == "loop.step":
            x = 0.5 * torch.randn(shape, generator=g)
        elif name == "embed":
            x = 0.4 * torch.randn(shape, generator=g)
        else:
            x = torch.randn(shape, generator=g) / math.sqrt(shape[-1])
        w[name] = x.to(torch.bfloat16).to(torch.float64).numpy()
    return w
