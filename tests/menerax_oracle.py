"""
A plain, slow float64 implementation of the Menerax design, written from its equations: one function per mechanism, token by token where the design is
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


def rms_unit(x, eps):
    """x over the root of its mean square (last axis), eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return rms_unit(x, eps) * w


def norm_around_zero(x, w, eps):
    """The model's norm: the stored weight is the deviation from one."""
    return rms_unit(x, eps) * (1.0 + w)


def pair_frequencies(rot):
    """Per pair i the angle of one position, base^(-2i / dims); with `scaling` slow pairs are slowed down further by `factor`, fast ones kept, and those between
    blended by how many turns the original context holds."""
    dims, base, sc = rot["dims"], float(rot["base"]), rot.get("scaling")
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc is not None:
            length = 2.0 * np.pi / f
            if length > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif length >= sc["original"] / sc["high"]:
                s = (sc["original"] / length - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate(x, positions, rot, interleaved):
    """x [T, ..., D]: the first rot.dims entries of the last axis turn with the position; pairs (2i, 2i + 1) or (i, i + dims / 2)."""
    out, dims = x.copy(), rot["dims"]
    for t, p in enumerate(positions):
        for i, f in enumerate(pair_frequencies(rot)):
            a = p * f
            iu, iv = (2 * i, 2 * i + 1) if interleaved else (i, i + dims // 2)
            u, v = x[t, ..., iu], x[t, ..., iv]
            out[t, ..., iu] = u * np.cos(a) - v * np.sin(a)
            out[t, ..., iv] = v * np.cos(a) + u * np.sin(a)
    return out


def softmax_read(q, k, v, scale, visible, softcap=None):
    """q [T, d], k [T, d], v [T, dv] of one head; visible(i, j) says whether row i sees key j."""
    T = q.shape[0]
    out = np.zeros((T, v.shape[1]))
    for i in range(T):
        js = [j for j in range(T) if visible(i, j)]
        s = (k[js] @ q[i]) * scale
        if softcap is not None:
            s = softcap * np.tanh(s / softcap)
        e = np.exp(s - s.max())
        out[i] = (e / e.sum()) @ v[js]
    return out


def kept_window(size, keep_first):
    return lambda i, j: j <= i and (i - j < size or j < keep_first)


def short_convolution(u, w):
    """u [T, C], w [C, taps]: row t = sum over i < taps of w[:, taps - 1 - i] u[t - i], nothing ahead of row 0."""
    taps = w.shape[1]
    out = np.zeros_like(u)
    for t in range(u.shape[0]):
        for j in range(taps):
            at = t - taps + 1 + j
            if at >= 0:
                out[t] += w[:, j] * u[at]
    return out


def latent_attention(h, W, pre, m, eps):
    H, d, r, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    T = h.shape[0]
    cq = rms_norm(h @ W[pre + "dq"].T, W[pre + "dq.norm"], eps)
    q = (cq @ W[pre + "uq"].T).reshape(T, H, d + r)
    z = h @ W[pre + "dkv"].T
    assert z.shape[1] == rank + r
    c = rms_norm(z[:, :rank], W[pre + "dkv.norm"], eps)
    qr, kr = rotate(q[:, :, d:], range(T), m["rot"], True), rotate(z[:, rank:], range(T), m["rot"], True)
    k = (c @ W[pre + "uk"].T).reshape(T, H, d)
    v = (c @ W[pre + "uv"].T).reshape(T, H, dv)
    gate = sigmoid(h @ W[pre + "g"].T)                          # one number per head
    heads = []
    for hd in range(H):
        qq = np.concatenate([q[:, hd, :d], qr[:, hd]], axis=1)
        kk = np.concatenate([k[:, hd], kr], axis=1)
        heads.append(softmax_read(qq, kk, v[:, hd], m["scale"], lambda i, j: j <= i) * gate[:, hd: hd + 1])
    return np.concatenate(heads, axis=1) @ W[pre + "o"].T


def window_attention(h, W, pre, m, eps):
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q, k, v = (short_convolution(h @ W[pre + nm].T + W[pre + nm + ".b"], W[pre + nm + ".conv"]) for nm in ("q", "k", "v"))
    q = rotate(rms_norm(q.reshape(T, H, d), W[pre + "q.norm"], eps), range(T), m["rot"], False)
    k = rotate(rms_norm(k.reshape(T, G, d), W[pre + "k.norm"], eps), range(T), m["rot"], False)
    v = v.reshape(T, G, dv)
    see = kept_window(m["mask"]["size"], m["mask"]["keep_first"])
    heads = [softmax_read(q[:, hd], k[:, hd // (H // G)], v[:, hd // (H // G)], m["scale"], see, m["softcap"]) for hd in range(H)]
    return (np.concatenate(heads, axis=1) * sigmoid(h @ W[pre + "g"].T)) @ W[pre + "o"].T


def shifted_mix(h, mu):
    """h_t + (h_(t-1) - h_t) mu, h_(-1) = 0."""
    before = np.concatenate([np.zeros((1, h.shape[1])), h[:-1]])
    return h + (before - h) * mu


def decay_of(z):
    return np.exp(-np.exp(z))


def time_mix_scan(r, k, v, w, u):
    """r, k, w [T, d], v [T, dv], u [d] of one head: o = S^T r + (r . (u k)) v, then row c of S times w_c, plus k_c v.  Returns o and the last S [d, dv]."""
    S = np.zeros((r.shape[1], v.shape[1]))
    out = np.zeros_like(v)
    for t in range(r.shape[0]):
        kv = np.outer(k[t], v[t])
        out[t] = (S + u[:, None] * kv).T @ r[t]
        S = w[t][:, None] * S + kv
    return out, S


def time_mixing(h, W, pre, m, eps):
    H, d = m["heads"], m["dim"]
    T = h.shape[0]
    mix = {nm: shifted_mix(h, W[pre + "mu." + nm]) for nm in "rkvgw"}
    r, k, v = ((mix[nm] @ W[pre + nm].T).reshape(T, H, d) for nm in "rkv")
    gate = silu(mix["g"] @ W[pre + "g"].T)
    w = decay_of(np.tanh(mix["w"] @ W[pre + "w1"].T) @ W[pre + "w2"].T + W[pre + "w0"]).reshape(T, H, d)
    o = np.concatenate([rms_unit(time_mix_scan(r[:, x], k[:, x], v[:, x], w[:, x], W[pre + "u"][x])[0], eps) for x in range(H)], axis=1)
    return (o * W[pre + "norm"] * gate) @ W[pre + "o"].T


def mixer(h, W, pre, L, eps):
    m = L["mixer"]
    if L["type"] == "latent_attention":
        return latent_attention(h, W, pre, m, eps)
    if L["type"] == "parallel":
        return m["left_scale"] * window_attention(h, W, pre + "left.", m["left"], eps) + m["right_scale"] * time_mixing(h, W, pre + "right.", m["right"], eps)
    raise ValueError(L["type"])


def feed_forward(h, W, pre, limit):
    g = np.minimum(h @ W[pre + "gate"].T, limit)
    u = np.clip(h @ W[pre + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ W[pre + "down"].T


def forward(cfg, W, tokens, taps_out=None):
    """tokens of ONE sequence -> logits [T, vocab] (float64).  taps_out: a list to which every layer appends the stream it leaves."""
    eps = float(cfg["norm"]["eps"])
    x = norm_around_zero(W["embed"][np.asarray(tokens)], W["embed.norm"], eps)
    for i, L in enumerate(cfg["layers"]):
        while L.get("weights_of") is not None:
            i = L["weights_of"]
            L = cfg["layers"][i]
        pre = f"l{i}."
        x = x + norm_around_zero(mixer(x, W, pre + "mix.", L, eps), W[pre + "norm1"], eps)
        if L.get("mlp") is not None:
            x = x + norm_around_zero(feed_forward(x, W, pre + "mlp.", L["mlp"]["limit"]), W[pre + "norm2"], eps)
        if taps_out is not None:
            taps_out.append(x.copy())
    return norm_around_zero(x, W["final.norm"], eps) @ W["head"].T
