"""
A plain, slow float64 implementation of the Luzinex design, written from its equations: one function per mechanism, token by token where the design is
recurrent and key by key in the masks, sharing no code with the product path.  Test infrastructure only.

Weights are a dict name -> float64 numpy array (the names a checkpoint uses); `cfg` is the parsed config.json.  Sequences are processed one at a
time and whole, so nothing here knows about steps, slots, pages or batches.
"""
from __future__ import annotations
import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def rms_unit(x, eps):
    """x over the root of its mean square (last axis)."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return rms_unit(x, eps) * w


def rotate(x, positions, dims, base, interleaved):
    """x [T, ..., D]: the first `dims` entries of the last axis turn with the position; pairs (2i, 2i + 1) or (i, i + dims / 2)."""
    out = x.copy()
    for t, p in enumerate(positions):
        for i in range(dims // 2):
            a = p * float(base) ** (-2.0 * i / dims)
            iu, iv = (2 * i, 2 * i + 1) if interleaved else (i, i + dims // 2)
            u, v = x[t, ..., iu], x[t, ..., iv]
            out[t, ..., iu] = u * np.cos(a) - v * np.sin(a)
            out[t, ..., iv] = v * np.cos(a) + u * np.sin(a)
    return out


def softmax_read(q, k, v, scale, visible, sink=None):
    """q [T, d], k [T, d], v [T, dv] of one head; visible(i, j) says whether row i sees key j; sink: a score without a key."""
    T = q.shape[0]
    out = np.zeros((T, v.shape[1]))
    for i in range(T):
        js = [j for j in range(T) if visible(i, j)]
        s = (k[js] @ q[i]) * scale
        top = s.max() if sink is None else max(s.max(), sink)
        e = np.exp(s - top)
        den = e.sum() + (0.0 if sink is None else np.exp(sink - top))
        out[i] = (e / den) @ v[js]
    return out


def latent_keys(h, W, pre, m, eps):
    """What a layer's cache holds: the normed latent c [T, rank] and the shared rotated key part [T, rot_dim]."""
    rank, r = m["kv_rank"], m["rot_dim"]
    z = h @ W[pre + "dkv"].T
    assert z.shape[1] == rank + r
    c = rms_norm(z[:, :rank], W[pre + "dkv.norm"], eps)
    return c, rotate(z[:, rank:], range(h.shape[0]), m["rot"]["dims"], m["rot"]["base"], False)


def latent_attention(h, W, pre, m, eps, c, kr):
    H, d, r, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    T = h.shape[0]
    cq = rms_norm(h @ W[pre + "dq"].T, W[pre + "dq.norm"], eps)
    q = (cq @ W[pre + "uq"].T).reshape(T, H, d + r)
    qr = rotate(q[:, :, d:], range(T), m["rot"]["dims"], m["rot"]["base"], False)
    k = (c @ W[pre + "uk"].T).reshape(T, H, d)
    v = (c @ W[pre + "uv"].T).reshape(T, H, dv)
    heads = []
    for hd in range(H):
        qq = np.concatenate([q[:, hd, :d], qr[:, hd]], axis=1)
        kk = np.concatenate([k[:, hd], kr], axis=1)
        heads.append(softmax_read(qq, kk, v[:, hd], m["scale"], lambda i, j: j <= i))
    o = np.concatenate(heads, axis=1) * sigmoid(h @ W[pre + "g"].T)
    return o @ W[pre + "o"].T


def kept_window(size, keep_first):
    return lambda i, j: j <= i and (i - j < size or j < keep_first)


def window_attention(h, W, pre, m):
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    T = h.shape[0]
    q = (h @ W[pre + "q"].T).reshape(T, H, d)
    v = (h @ W[pre + "k"].T).reshape(T, G, d)                  # the values are the keys before their rotation
    rot = m["rot"]
    q, k = (rotate(t, range(T), rot["dims"], rot["base"], True) for t in (q, v))
    see = kept_window(m["mask"]["size"], m["mask"]["keep_first"])
    heads = [softmax_read(q[:, hd], k[:, hd // (H // G)], v[:, hd // (H // G)], m["scale"], see, W[pre + "sink"][hd]) for hd in range(H)]
    o = np.concatenate(heads, axis=1) * sigmoid(h @ W[pre + "g"].T)
    return o @ W[pre + "o"].T


def retention_scan(q, k, v, decay):
    """q, k [T, d], v [T, dv] of one head: S <- decay S + k v^T, o = S^T q.  Returns o and the last S [d, dv]."""
    S = np.zeros((q.shape[1], v.shape[1]))
    out = np.zeros_like(v)
    for t in range(q.shape[0]):
        S = decay * S + np.outer(k[t], v[t])
        out[t] = S.T @ q[t]
    return out, S


def retention(h, W, pre, m, eps):
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    rot = m["rot"]
    q, k = (rotate((h @ W[pre + nm].T).reshape(T, H, d), range(T), rot["dims"], rot["base"], False) for nm in ("q", "k"))
    k = k * d ** -0.5
    v = (h @ W[pre + "v"].T).reshape(T, H, dv)
    o = np.concatenate([rms_unit(retention_scan(q[:, hd], k[:, hd], v[:, hd], m["decay"][hd])[0], eps) for hd in range(H)], axis=1)
    return (o * silu(h @ W[pre + "g"].T)) @ W[pre + "o"].T


def feed_forward(h, W, pre):
    return (gelu_tanh(h @ W[pre + "gate"].T) * (h @ W[pre + "up"].T)) @ W[pre + "down"].T


def forward(cfg, W, tokens, taps_out=None):
    """tokens of ONE sequence -> logits [T, vocab] (float64).  taps_out: a list that receives the residual stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][np.asarray(tokens)]
    held = {}
    for i, L in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", L["mixer"]
        h = rms_norm(x, W[pre + "norm1"], eps)
        if L["type"] == "latent_attention":
            src = m.get("kv_from")
            if src is None:
                held[i] = latent_keys(h, W, pre + "mix.", m, eps)
                src = i
            y = latent_attention(h, W, pre + "mix.", m, eps, *held[src])
        elif L["type"] == "attention":
            y = window_attention(h, W, pre + "mix.", m)
        elif L["type"] == "retention":
            y = retention(h, W, pre + "mix.", m, eps)
        else:
            raise ValueError(L["type"])
        if L.get("mlp") is not None:
            y = y + feed_forward(rms_norm(x, W[pre + "norm2"], eps), W, pre + "mlp.")
        x = x + y
        if taps_out is not None:
            taps_out.append(x.copy())
    return rms_norm(x, W["final.norm"], eps) @ W["head"].T
