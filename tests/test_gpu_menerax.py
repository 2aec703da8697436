"""GPU tests of the Menerax design (csrc/mix_timemix.hip, csrc/mix_convprep.hip, the post-norm update and the embedding norm of mix_rowops.hip, gates per head, factors on
attention results, modules.py, menerax.py) against the float64 oracle of tests/menerax_oracle.py: every mechanism alone, whole models of several small shapes (written to a
checkpoint folder and loaded through the registry), prefill against token-by-token decoding, unequal batches against each request alone, slots and pages that are freed and
used again, one dominant key at every edge of a window, the first tokens, long decoding, trace replay and greedy generation through the scheduler.  float32 runs are held
to float32 rounding; bfloat16 runs to a loose bar (the oracle does not round)."""
import io
import json
import math
import os
from types import SimpleNamespace
import numpy as np
import pytest
import torch
import menerax_oracle as mo

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 3e-5, torch.bfloat16: 4e-2}
VOCAB = 83


@pytest.fixture(scope="module")
def gpu():
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    from exllamav3_amd import _lib
    _lib.mixlib()
    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")
    return torch.device("cuda:0")


def npy(t):
    return t.detach().double().cpu().numpy()


def rel(a, b):
    a = npy(a) if isinstance(a, torch.Tensor) else np.asarray(a, dtype=np.float64)
    b = npy(b) if isinstance(b, torch.Tensor) else np.asarray(b, dtype=np.float64)
    assert a.shape == b.shape
    return float(np.abs(a - b).max() / (np.abs(b).max() + 1e-30))


def mk(gpu, v):
    return torch.tensor(v, dtype=torch.int32, device=gpu)


def step_of(gpu, lens, pos0=None, slots=None):
    """The row tensors of a packed step."""
    pos0 = pos0 or [0] * len(lens)
    slots = slots or list(range(len(lens)))
    cu = [0]
    for l in lens: cu.append(cu[-1] + l)
    seq = [i for i, l in enumerate(lens) for _ in range(l)]
    pos = [pos0[i] + j for i, l in enumerate(lens) for j in range(l)]
    return SimpleNamespace(n=cu[-1], cu=mk(gpu, cu), tok_seq=mk(gpu, seq), tok_pos=mk(gpu, pos), slots=mk(gpu, slots), pos0=mk(gpu, pos0),
                           len_after=mk(gpu, [p + l for p, l in zip(pos0, lens)]), max_rows=max(lens))


def freqs(gpu, rot):
    from exllamav3_amd.modules import rotary_frequencies
    return rotary_frequencies(rot["dims"], rot["base"], rot.get("scaling"))[0].to(gpu).contiguous() if rot["dims"] else None


# ---- the mechanisms alone -----------------------------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [37, 72, 1032])
def test_embedding_with_its_norm(gpu, dtype, width):
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(width)
    table, w, toks = (2 * torch.randn(11, width, generator=g)).to(dtype), 0.3 * torch.randn(width, generator=g), [3, 0, 10, 3]
    x, h = torch.empty(4, width, device=gpu), torch.full((4, width + 8), 5.0, dtype=dtype, device=gpu)
    mix_ops.embed_norm(x, h[:, :width], table.to(gpu), mk(gpu, toks), (1 + w).to(gpu), 1e-3)
    want = mo.norm_around_zero(npy(table)[toks], npy(w), 1e-3)
    assert rel(x, want) < 1e-6 and rel(h[:, :width], want) < TOL[dtype] / 4 and bool((h[:, width:] == 5.0).all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [33, 68, 1028, 4100, 6000])
def test_residual_update_with_a_normed_addend(gpu, dtype, width):
    """Rows of a few elements up to rows longer than what a workgroup keeps in registers; aligned and unaligned addends."""
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(width)
    n = 5
    w = 0.3 * torch.randn(width, generator=g)
    for pad, off in ((8, 0), (8, 1), (3, 0)):
        x, y = torch.randn(n, width, generator=g), (0.02 * torch.randn(n, width + pad, generator=g)).to(dtype)       # small rows: eps matters
        xd, yd = x.to(gpu), y.to(gpu)[:, off: off + width]
        h = torch.full((n, width + 8), 3.0, dtype=dtype, device=gpu)
        mix_ops.residual_norm(xd, yd, mix_ops.RES_ADD, (1 + w).to(gpu), 1e-3, mix_ops.OUT_CAST, 0.0, None, None, h[:, :width])
        want = npy(x) + mo.norm_around_zero(npy(y)[:, off: off + width], npy(w), 1e-3)
        assert rel(xd, want) < 1e-6 and rel(h[:, :width], want) < TOL[dtype] / 4 and bool((h[:, width:] == 3.0).all())
        xd = x.to(gpu)
        mix_ops.residual_norm(xd, yd, mix_ops.RES_ADD, (1 + w).to(gpu), 1e-3, mix_ops.OUT_NONE, 0.0, None, None, None)
        assert rel(xd, want) < 1e-6


@pytest.mark.parametrize("dtype", DTYPES)
def test_gate_per_head_and_per_element(gpu, dtype):
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(2)
    n, H, dv = 5, 3, 12
    a, gh, ge = torch.randn(H, n, dv, generator=g).to(dtype), torch.randn(n, H + 5, generator=g).to(dtype), torch.randn(n, H * dv, generator=g).to(dtype)
    base = npy(a).transpose(1, 0, 2)
    for gate, want in ((gh.to(gpu)[:, 2: 2 + H], base * mo.sigmoid(npy(gh)[:, 2: 2 + H])[:, :, None]), (ge.to(gpu), base * mo.sigmoid(npy(ge)).reshape(n, H, dv)), (None, base)):
        o = torch.empty(n, H * dv, dtype=dtype, device=gpu)
        mix_ops.heads_gate(o, a.to(gpu), dv, n * dv, gate, H, dv)
        assert rel(o, want.reshape(n, -1)) < TOL[dtype] / 4


ROT = {"dims": 8, "base": 5000.0, "scaling": {"factor": 4.0, "low": 1.0, "high": 3.0, "original": 64}}


def attend(gpu, dtype, u, conv, qn, kn, gate, m, lens, decode_from, slots, eps=1e-4, out_scale=1.0, mfma=None):
    """Convolution, norms, rotation, cache store and attention for sequences of projected rows u [T, C]: the first decode_from[i] rows as one packed prompt step, the rest token
    by token.  Returns per sequence [T, H * dv]."""
    from exllamav3_amd import mix_ops
    H, G, d, dv, size, keep, scale, cap = (m[k] for k in ("heads", "kv_heads", "dim", "vdim", "size", "keep", "scale", "softcap"))
    taps, C = conv.shape
    rk = torch.full((max(slots) + 2, keep + size, G, d), float("nan"), dtype=dtype, device=gpu)
    rv = torch.full((max(slots) + 2, keep + size, G, dv), float("nan"), dtype=dtype, device=gpu)
    ring = torch.full((max(slots) + 2, max(taps - 1, 1), C), float("nan"), dtype=dtype, device=gpu)
    freq = freqs(gpu, m["rot"])
    dev = lambda t: None if t is None else t.to(gpu)
    outs = [[] for _ in lens]

    def step(lo_, hi_):
        live = [i for i in range(len(lens)) if hi_[i] > lo_[i]]
        ln = [hi_[i] - lo_[i] for i in live]
        sb = step_of(gpu, ln, [lo_[i] for i in live], [slots[i] for i in live])
        pick = lambda t: torch.cat([t[i][lo_[i]: hi_[i]] for i in live]).to(dtype)
        wide = torch.cat([pick(u), pick(gate)], dim=1).to(gpu)                    # the column blocks of one wide product, as a model has them
        z = torch.empty(sb.n, C, dtype=dtype, device=gpu)
        mix_ops.conv_prep(z, wide[:, :C], conv.to(gpu), ring, dev(qn), dev(kn), freq, 1.0, False, eps, rk, rv, sb, H, keep_first=keep)
        q, k, v, gv = z[:, : H * d], z[:, H * d: (H + G) * d], z[:, (H + G) * d:], wide[:, C:]
        wide_out = torch.full((sb.n, H * dv + 8), 3.0, dtype=dtype, device=gpu)
        out = wide_out[:, : H * dv]
        if lo_[live[0]] == 0:
            mix_ops.attn_prefill_maps(out, q, k, v, gv, None, sb.cu, sb.tok_seq, sb.tok_pos, H, G, 1, d, dv, scale, cap, size, mix_ops.MASK_WINDOW, max_rows=max(ln), keep=keep,
                                      mfma=mfma, out_scale=out_scale)
        else:
            mix_ops.attn_decode_maps(out, q, rk, rv, gv, None, sb.slots, sb.len_after, H, 1, scale, cap, mix_ops.MASK_WINDOW, out_scale=out_scale)
        assert bool((wide_out[:, H * dv:] == 3.0).all())
        at = 0
        for i, l in zip(live, ln):
            outs[i].append(npy(out[at: at + l])); at += l

    step([0] * len(lens), decode_from)
    done = list(decode_from)
    while any(a < l for a, l in zip(done, lens)):
        nxt = [min(a + 1, l) for a, l in zip(done, lens)]
        step(done, nxt); done = nxt
    return [np.concatenate(o) for o in outs]


def attend_truth(u, conv, qn, kn, gate, m, dtype, eps=1e-4, out_scale=1.0):
    H, G, d, dv = (m[k] for k in ("heads", "kv_heads", "dim", "vdim"))
    u, gate, T = npy(u.to(dtype)), npy(gate.to(dtype)), u.shape[0]
    y = mo.short_convolution(u, npy(conv).T)
    q, k, v = y[:, : H * d].reshape(T, H, d), y[:, H * d: (H + G) * d].reshape(T, G, d), y[:, (H + G) * d:].reshape(T, G, dv)
    q, k = (t if w is None else mo.rms_norm(t, npy(w), eps) for t, w in ((q, qn), (k, kn)))
    q, k = (mo.rotate(t, range(T), m["rot"], False) for t in (q, k))
    see = mo.kept_window(m["size"], m["keep"])
    o = np.concatenate([mo.softmax_read(q[:, h], k[:, h // (H // G)], v[:, h // (H // G)], m["scale"], see, m["softcap"] or None) for h in range(H)], axis=1)
    return out_scale * o * mo.sigmoid(gate)


ATTENTION = [  # heads, kv_heads, dim, vdim, size, keep, softcap, taps, rotated, normed
    (4, 2, 16, 24, 9, 3, 20.0, 4, 8, True),
    (2, 2, 24, 16, 33, 1, 3.0, 2, 24, True),
    (3, 1, 10, 7, 5, 0, 15.0, 3, 4, True),                      # no vector access fits
    (6, 2, 64, 48, 70, 66, 30.0, 4, 32, True),                  # the sizes of the matrix-core kernel
    (1, 1, 8, 8, 1, 2, 5.0, 1, 2, True),                        # a window of one, one tap
    (2, 1, 72, 40, 64, 64, 0.0, 5, 0, True),                    # no cap, no rotation, more taps than the unrolled forms
    (5, 5, 128, 128, 40, 0, 25.0, 3, 64, False),
    (17, 1, 64, 64, 12, 5, 9.0, 4, 64, True),                   # more heads than one group of a workgroup
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", ATTENTION)
def test_window_attention_prompts_and_decoding(gpu, dtype, shape):
    H, G, d, dv, size, keep, cap, taps, dims, normed = shape
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "size": size, "keep": keep, "softcap": cap, "scale": 1.7 / math.sqrt(d), "rot": dict(ROT, dims=dims)}
    g = torch.Generator().manual_seed(size + d)
    lens, first = [150, 41, keep + 2, 3], [110, 37, keep + 1, 1]
    C = (H + G) * d + G * dv
    u, gate = [torch.randn(l, C, generator=g) for l in lens], [torch.randn(l, H * dv, generator=g) for l in lens]
    conv = 0.6 * torch.randn(taps, C, generator=g)
    qn, kn = (torch.rand(d, generator=g) + 0.5 if normed else None for _ in range(2))
    got = attend(gpu, dtype, u, conv, qn, kn, gate, m, lens, first, [2, 0, 1, 4], out_scale=1.3)
    for i in range(len(lens)):
        assert rel(got[i], attend_truth(u[i], conv, qn, kn, gate[i], m, dtype, out_scale=1.3)) < TOL[dtype], i


@pytest.mark.parametrize("dtype", DTYPES)
def test_convolved_rows_of_a_long_packed_step(gpu, dtype):
    """Enough rows for the form that keeps the convolution's weights over several of them, with sequence borders inside its groups of rows."""
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(8)
    lens, H, G, d, dv, taps, size, keep = [1, 2, 301, 3, 250, 5], 3, 1, 16, 24, 4, 20, 2
    C, eps = (H + G) * d + G * dv, 1e-4
    u, conv = [torch.randn(l, C, generator=g).to(dtype) for l in lens], torch.randn(taps, C, generator=g)
    qn, kn = torch.rand(d, generator=g) + 0.5, torch.rand(d, generator=g) + 0.5
    sb = step_of(gpu, lens)
    assert sb.n >= 512
    rk, rv = torch.full((6, keep + size, G, d), float("nan"), dtype=dtype, device=gpu), torch.full((6, keep + size, G, dv), float("nan"), dtype=dtype, device=gpu)
    ring = torch.full((6, taps - 1, C), float("nan"), dtype=dtype, device=gpu)
    z = torch.empty(sb.n, C, dtype=dtype, device=gpu)
    mix_ops.conv_prep(z, torch.cat(u).to(gpu), conv.to(gpu), ring, qn.to(gpu), kn.to(gpu), freqs(gpu, ROT), 1.0, False, eps, rk, rv, sb, H, keep_first=keep)
    at = 0
    for i, l in enumerate(lens):
        y = mo.short_convolution(npy(u[i]), npy(conv).T)
        q = mo.rotate(mo.rms_norm(y[:, : H * d].reshape(l, H, d), npy(qn), eps), range(l), ROT, False).reshape(l, -1)
        k = mo.rotate(mo.rms_norm(y[:, H * d: (H + G) * d].reshape(l, G, d), npy(kn), eps), range(l), ROT, False).reshape(l, -1)
        v = y[:, (H + G) * d:]
        for a, b in ((z[at: at + l, : H * d], q), (z[at: at + l, H * d: (H + G) * d], k), (z[at: at + l, (H + G) * d:], v)):
            assert rel(a, b) < (1e-4 if dtype == torch.float32 else 1e-2), i                        # float32 angles at position 300
        for e in range(min(l, keep + size)):                        # which position an entry holds
            p = e if e < keep else max(x for x in range(keep, l) if keep + (x - keep) % size == e)
            assert rel(rk[i, e].reshape(-1), k[p]) < 1e-2 and rel(rv[i, e].reshape(-1), v[p]) < 1e-2, (i, e)
        for p in range(max(0, l - taps + 1), l):
            assert torch.equal(ring[i, p % (taps - 1)].float().cpu(), u[i][p].float())              # the projected rows as they are
        at += l


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("size,keep,T", [(40, 5, 300), (64, 64, 260), (1, 3, 90), (37, 0, 200)])
def test_one_key_stands_out_at_every_edge_of_the_window(gpu, dtype, decoded, size, keep, T):
    """Row i = T - 1 and one loud key at j: in sight it takes nearly all the weight, out of sight it must leave no trace."""
    d, dv, i = 16, 16, T - 1
    m = {"heads": 1, "kv_heads": 1, "dim": d, "vdim": dv, "size": size, "keep": keep, "softcap": 20.0, "scale": 0.25, "rot": ROT}
    conv = torch.zeros(3, 2 * d + dv)
    conv[2] = 1.0                                                    # queries, keys and values as projected
    big = torch.full((d,), 3.0)
    for j in sorted({0, max(keep - 1, 0), keep, keep + 1, i - size - 1, i - size, i - size + 1, i - size + 2, i - 1, i, T // 2}):
        if not 0 <= j <= i:
            continue
        g = torch.Generator().manual_seed(j)
        u, gate = torch.randn(T, 2 * d + dv, generator=g), torch.randn(T, dv, generator=g)
        u[:, 2 * d - 1] = 0.0                                        # no key reaches into the last entry (beyond the rotated ones) ...
        u[i, :d] = 0.0; u[i, d - 1] = 1.0                            # ... in which alone row i asks
        u[j, d: 2 * d] = 0.0; u[j, 2 * d - 1] = 1.0
        u[:, 2 * d], u[j, 2 * d] = 0.0, 9.0
        got = attend(gpu, dtype, [u], conv, big, big, [gate], m, [T], [T - 3 if decoded else T], [0])[0]
        want = attend_truth(u, conv, big, big, gate, m, dtype)
        assert rel(got[i], want[i]) < TOL[dtype], j
        seen = i - j < size or j < keep
        assert (np.abs(want[i, 0] / mo.sigmoid(npy(gate)[i, 0])) > 8.0) == seen and (seen or np.abs(got[i, 0]) < 1e-6), j


@pytest.mark.parametrize("mfma", [False, True])
def test_the_cap_bounds_scores_on_both_paths(gpu, mfma):
    """Scores far beyond the cap: weights are at most e^(2 cap) apart."""
    T, d, dv = 90, 32, 32
    m = {"heads": 2, "kv_heads": 1, "dim": d, "vdim": dv, "size": 50, "keep": 4, "softcap": 2.0, "scale": 3.0, "rot": ROT}
    g = torch.Generator().manual_seed(3)
    u, gate, conv = torch.randn(T, 3 * d + dv, generator=g), torch.randn(T, 2 * dv, generator=g), torch.randn(4, 3 * d + dv, generator=g)
    qn = torch.full((d,), 2.0)
    got = attend(gpu, torch.bfloat16, [u], conv, qn, qn, [gate], m, [T], [T], [0], mfma=mfma)[0]
    assert rel(got, attend_truth(u, conv, qn, qn, gate, m, torch.bfloat16)) < 4e-2
    assert rel(attend_truth(u, conv, qn, qn, gate, dict(m, softcap=None), torch.bfloat16), got) > 0.3


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [40, 37, 2056])
@pytest.mark.parametrize("lens", [[5, 1, 2], [700, 1, 330, 2]])
def test_token_shift(gpu, dtype, width, lens):
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(width)
    slots, mu = list(range(len(lens)))[::-1], torch.rand(5, width, generator=g)
    h = [torch.randn(l + 2, width, generator=g).to(dtype) for l in lens]
    want = [np.stack([mo.shifted_mix(npy(t), npy(mu[m])) for m in range(5)]) for t in h]
    last = torch.full((len(lens) + 1, width), float("nan"), dtype=dtype, device=gpu)
    done = [0] * len(lens)
    for nxt in (lens, [l + 1 for l in lens], [l + 2 for l in lens]):
        sb = step_of(gpu, [b - a for a, b in zip(done, nxt)], done, slots)
        out = torch.full((5, sb.n, width), float("nan"), dtype=dtype, device=gpu)
        wide = torch.cat([t[a:b] for t, a, b in zip(h, done, nxt)]).to(gpu)
        mix_ops.token_shift(out, wide, last, mu.to(gpu), sb)
        assert rel(out, np.concatenate([w[:, a:b] for w, a, b in zip(want, done, nxt)], axis=1)) < TOL[dtype] / 4
        for t, s, b in zip(h, slots, nxt):
            assert torch.equal(last[s].cpu(), t[b - 1])
        done = list(nxt)
    assert torch.isnan(last[-1]).all()


@pytest.mark.parametrize("n", [1, 4, 5, 16])
@pytest.mark.parametrize("rows,K", [(37, 40), (16, 8), (64, 4104), (1000, 264), (8200, 1032), (20, 32)])
def test_products_of_few_rows(gpu, n, rows, K):
    """Heights and depths that no tile fits, a bias, weights and rows that are column blocks of wider matrices."""
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(rows + K + n)
    bf = torch.bfloat16
    x, w, b = torch.randn(n, K + 16, generator=g).to(bf), (torch.randn(rows, K + 8, generator=g) / math.sqrt(K)).to(bf), torch.randn(rows, generator=g).to(bf)
    for xv, wv, bias in ((x[:, 8: 8 + K], w[:, :K], b), (x[:, :K].contiguous(), w[:, 8:].contiguous(), None)):
        ref = npy(xv) @ npy(wv).T + (npy(b) if bias is not None else 0.0)
        xd, wd = (xv if xv.is_contiguous() else None), None
        xd = x.to(gpu)[:, 8: 8 + K] if xd is None else xd.to(gpu)
        wd = wv.to(gpu) if wv.is_contiguous() else w.to(gpu)[:, :K]
        assert mix_ops.skinny_ok(xd, wd)
        assert rel(mix_ops.skinny(xd, wd, None if bias is None else b.to(gpu)), ref) < 8e-3
    assert not mix_ops.skinny_ok(torch.zeros(17, 16, dtype=bf, device=gpu), torch.zeros(4, 16, dtype=bf, device=gpu))
    assert not mix_ops.skinny_ok(torch.zeros(2, 12, dtype=bf, device=gpu), torch.zeros(4, 12, dtype=bf, device=gpu)) and not mix_ops.skinny_ok(torch.zeros(2, 16, device=gpu), torch.zeros(4, 16, device=gpu))


@pytest.mark.parametrize("n", [1, 3, 16])
@pytest.mark.parametrize("mats,rows,tail,K", [(4, 48, 16, 40), (4, 33, 5, 264), (2, 4112, 70, 96), (1, 7, 3, 8)])
def test_stacked_products_of_few_rows(gpu, n, mats, rows, tail, K):
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(rows + n)
    x, w = torch.randn(mats + 1, n, K, generator=g).to(torch.bfloat16), (torch.randn(mats * rows + tail, K, generator=g) / math.sqrt(K)).to(torch.bfloat16)
    y, t = mix_ops.skinny_stack(x.to(gpu), w.to(gpu), rows)
    for m in range(mats):
        assert rel(y[m], npy(x[m]) @ npy(w[m * rows: (m + 1) * rows]).T) < 8e-3
    assert rel(t, npy(x[mats]) @ npy(w[mats * rows:]).T) < 8e-3


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,channels,rank", [(3, 48, 16), (70, 300, 64), (33, 21, 5), (200, 512, 40), (17, 260, 136)])
def test_decay_logarithms(gpu, dtype, n, channels, rank):
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(rank)
    t, w2, w0 = torch.randn(n, rank + 8, generator=g).mul(1.5).to(dtype), (torch.randn(channels, rank, generator=g) / math.sqrt(rank)).to(dtype), torch.randn(channels, generator=g) * 2 - 1
    out = torch.empty(n, channels, device=gpu)
    mix_ops.decay_log2(out, t.to(gpu)[:, :rank], w2.to(gpu), w0.to(gpu))
    want = np.log2(np.e) * -np.exp(np.tanh(npy(t)[:, :rank]) @ npy(w2).T + npy(w0))
    assert np.abs(npy(out) / want - 1).max() < 5e-6                              # float32 in both modes


DECAYS = {"usual": (-2.0, 1.5), "strong": (2.0, 1.5), "none": (-60.0, 0.0), "at once": (12.0, 0.0), "mixed": (0.0, 4.0)}


# heads, key and value sizes, segments; the sizes that no vector access fits run with mixed decays alone
TIME_MIX = [(2, 32, 32, None), (3, 64, 64, (3, 64)), (1, 48, 48, (5, 32)), (2, 7, 5, None), (1, 128, 72, (2, 80)), (2, 200, 33, (3, 48)), (1, 96, 96, None), (2, 64, 130, (4, 48))]
TIME_MIX_CASES = [(*shape, decays) for shape in TIME_MIX for decays in DECAYS if decays == "mixed" or shape[1] not in (7, 96, 200)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,dv,segments,decays", TIME_MIX_CASES)
def test_time_mixing_prompt_then_decoding(gpu, dtype, H, d, dv, segments, decays):
    """Any decays: from a state that forgets nothing to one that forgets everything at once, and channels of both kinds in one tile."""
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(d + dv)
    lens, extra, slots, rank = [125, 32, 1, 33], 3, [3, 1, 4, 0], 8
    mean, sd = DECAYS[decays]
    r, k = ([torch.randn(l + extra, H * d, generator=g).to(dtype) for l in lens] for _ in range(2))
    v, gt = ([torch.randn(l + extra, H * dv, generator=g).to(dtype) for l in lens] for _ in range(2))
    t = [torch.randn(l + extra, rank, generator=g).to(dtype) for l in lens]
    w2, w0 = (sd * torch.randn(H * d, rank, generator=g) / math.sqrt(rank)).to(dtype), mean + 0.5 * sd * torch.randn(H * d, generator=g)
    u, nw = torch.randn(H * d, generator=g), torch.rand(H * dv, generator=g) + 0.5
    want, last = [], []
    for i, l in enumerate(lens):
        T = l + extra
        w = mo.decay_of(np.tanh(npy(t[i])) @ npy(w2).T + npy(w0)).reshape(T, H, d)
        o = [mo.time_mix_scan(npy(r[i]).reshape(T, H, d)[:, h], npy(k[i]).reshape(T, H, d)[:, h], npy(v[i]).reshape(T, H, dv)[:, h], w[:, h], npy(u).reshape(H, d)[h]) for h in range(H)]
        want.append(np.stack([a for a, _ in o], axis=1)); last.append(np.stack([S for _, S in o]))
    heads = lambda i, lo_, hi_: ((mo.rms_unit(want[i][lo_:hi_], 1e-5).reshape(hi_ - lo_, -1) * npy(nw)) * mo.silu(npy(gt[i][lo_:hi_])))
    cat = lambda ts, lo_, hi_: torch.cat([x[a:b] for x, a, b in zip(ts, lo_, hi_)]).to(gpu)
    zero = [0] * len(lens)
    sb = step_of(gpu, lens, None, slots)
    log2w = torch.empty(sb.n, H * d, device=gpu)
    mix_ops.decay_log2(log2w, cat(t, zero, lens), w2.to(gpu), w0.to(gpu))
    tol = 3e-5
    for fused in ([False, True] if dv <= mix_ops.TIMEMIX_FUSED_VDIM else [False]):
        state = torch.full((6, H, d, dv), float("nan"), device=gpu)
        o = None if fused else torch.full((sb.n, H, dv), float("nan"), device=gpu)
        wide_out = torch.full((sb.n, H * dv + 8), 2.0, dtype=dtype, device=gpu)
        mix_ops.timemix(o, wide_out[:, : H * dv] if fused else None, cat(gt, zero, lens) if fused else None, nw.to(gpu), 1e-5, state, cat(r, zero, lens), cat(k, zero, lens),
                        cat(v, zero, lens), log2w, u.to(gpu), sb.cu, sb.slots, sb.pos0, segments=segments)
        at = 0
        for i, l in enumerate(lens):
            if fused: assert rel(wide_out[at: at + l, : H * dv], heads(i, 0, l)) < (1e-4 if dtype == torch.float32 else 1e-2), i
            else: assert rel(o[at: at + l], want[i][:l]) < tol, i                      # float32 in both modes: the inputs are what they are
            at += l
        assert bool((wide_out[:, H * dv:] == 2.0).all()) and torch.isnan(state[2]).all() and torch.isnan(state[5]).all()
    for x in range(extra):
        lo_, hi_ = [l + x for l in lens], [l + x + 1 for l in lens]
        wide_out = torch.full((len(lens), H * dv + 8), 2.0, dtype=dtype, device=gpu)
        mix_ops.timemix_step(wide_out[:, : H * dv], state, *(cat(y, lo_, hi_) for y in (r, k, v, gt, t)), w2.to(gpu), w0.to(gpu), u.to(gpu),
                             nw.to(gpu), mk(gpu, lo_), sb.slots, 1e-5)
        assert rel(wide_out[:, : H * dv], np.concatenate([heads(i, a, b) for i, (a, b) in enumerate(zip(lo_, hi_))])) < (1e-4 if dtype == torch.float32 else 1e-2), x
        assert bool((wide_out[:, H * dv:] == 2.0).all())
    for i in range(len(lens)):
        assert rel(state[slots[i]], last[i]) < tol


@pytest.mark.parametrize("dtype", DTYPES)
def test_time_mixing_from_the_first_token_by_steps_alone(gpu, dtype):
    """A sequence that is decoded from its first token starts from zero, whatever its slot held."""
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(1)
    H, d, T = 2, 24, 9
    r, k, v, gt = (torch.randn(T, H * d, generator=g).to(dtype) for _ in range(4))
    t, w2, w0 = torch.randn(T, 12, generator=g).to(dtype), torch.randn(H * d, 12, generator=g).to(dtype), torch.randn(H * d, generator=g) - 2
    u, nw = torch.randn(H * d, generator=g), torch.rand(H * d, generator=g)
    w = mo.decay_of(np.tanh(npy(t)) @ npy(w2).T + npy(w0)).reshape(T, H, d)
    sp = lambda x: npy(x).reshape(T, H, d)
    o = np.stack([mo.time_mix_scan(sp(r)[:, h], sp(k)[:, h], sp(v)[:, h], w[:, h], npy(u).reshape(H, d)[h])[0] for h in range(H)], axis=1)
    want = mo.rms_unit(o, 1e-5).reshape(T, -1) * npy(nw) * mo.silu(npy(gt))
    state = torch.full((2, H, d, d), float("nan"), device=gpu)
    for i in range(T):
        out, row = torch.empty(1, H * d, dtype=dtype, device=gpu), lambda x: x[i: i + 1].to(gpu)
        mix_ops.timemix_step(out, state, row(r), row(k), row(v), row(gt), row(t), w2.to(gpu), w0.to(gpu), u.to(gpu), nw.to(gpu), mk(gpu, [i]), mk(gpu, [1]), 1e-5)
        assert rel(out, want[i: i + 1]) < (1e-4 if dtype == torch.float32 else 1e-2), i


class Tensors:
    def __init__(self, t):
        self.t = t

    def get_tensor(self, key, device="cpu"):
        return self.t[key]


def mixer_case(gpu, dtype, L, width, seed, page=64):
    """One mixer with random weights over a cache of its own."""
    from exllamav3_amd.menerax import MeneraxConfig
    from exllamav3_amd.state_cache import SlotStateCache
    cfg = {"architecture": "Menerax", "vocab": 5, "width": width, "norm": {"eps": 1e-5}, "layers": [dict(L, mlp=None)]}
    W = {k: v.float() for k, v in weights(cfg, seed).items()}
    mx = MeneraxConfig(cfg).build_blocks()[0].mixer
    mx.load(Tensors(W), "l0.mix.", dtype, gpu)
    return cfg["layers"][0], {k: npy(v) for k, v in W.items()}, mx, SlotStateCache([mx.state_specs()], gpu, slots=4, page_size=page)


def par(left, right, ff=None, ls=0.8, rs=1.4, conv=4, cap=20.0, base=9000.0, limit=1.5, scaling=None, rank=6, **kw):
    """left: heads, kv_heads, dim, vdim, rotated, size, keep_first; right: heads, dim."""
    H, G, d, dv, dims, size, keep = left
    m = {"left": {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "conv": conv, "scale": 1.0 / math.sqrt(d), "softcap": cap, "mask": {"size": size, "keep_first": keep},
                  "rot": {"base": base, "dims": dims, "scaling": scaling or {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 128}}},
         "right": {"heads": right[0], "dim": right[1]}, "left_scale": ls, "right_scale": rs}
    return {"type": "parallel", "mixer": m, "mlp": ff and {"kind": "dense", "ff": ff, "limit": limit}, "_rank": rank}


def lat(heads, dim, rot, vdim, rank, q_rank, ff=None, base=30000.0, limit=1.5):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank, "scale": 1.0 / math.sqrt(dim + rot), "rot": {"base": base, "dims": rot}}
    return {"type": "latent_attention", "mixer": m, "mlp": ff and {"kind": "dense", "ff": ff, "limit": limit}}


def weights(cfg, seed):
    g = torch.Generator().manual_seed(seed)
    w, W = cfg["width"], {}

    def lin(name, o, i, s=1.0):
        W[name] = (s * torch.randn(o, i, generator=g) / math.sqrt(i)).to(torch.bfloat16)

    def vec(name, n, mean=0.0, s=0.3):
        W[name] = (mean + s * torch.randn(n, generator=g)).to(torch.bfloat16)
    W["embed"] = torch.randn(cfg["vocab"], w, generator=g).to(torch.bfloat16)
    vec("embed.norm", w); vec("final.norm", w)
    for i, L in enumerate(cfg["layers"]):
        if "weights_of" in L:
            continue
        m, p = L["mixer"], f"l{i}.mix."
        vec(f"l{i}.norm1", w)
        if L["type"] == "latent_attention":
            H, d, r, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            lin(p + "dq", m["q_rank"], w); vec(p + "dq.norm", m["q_rank"], 1.0); lin(p + "uq", H * (d + r), m["q_rank"])
            lin(p + "dkv", rank + r, w); vec(p + "dkv.norm", rank, 1.0)
            lin(p + "uk", H * d, rank); lin(p + "uv", H * dv, rank); lin(p + "g", H, w); lin(p + "o", w, H * dv)
        else:
            a, b, taps = m["left"], m["right"], m["left"]["conv"]
            q = p + "left."
            for nm, n in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
                lin(q + nm, n, w); vec(q + nm + ".b", n)
                W[q + nm + ".conv"] = (0.6 * torch.randn(n, taps, generator=g)).to(torch.bfloat16)
            vec(q + "q.norm", a["dim"], 1.0); vec(q + "k.norm", a["dim"], 1.0); lin(q + "g", a["heads"] * a["vdim"], w); lin(q + "o", w, a["heads"] * a["vdim"])
            q, n, rank = p + "right.", b["heads"] * b["dim"], L.get("_rank", 6)
            for nm in "rkvg":
                lin(q + nm, n, w)
            for nm in "rkvgw":
                W[q + "mu." + nm] = torch.rand(w, generator=g).to(torch.bfloat16)
            lin(q + "w1", rank, w); lin(q + "w2", n, rank); vec(q + "w0", n, -1.5, 1.0)
            W[q + "u"] = torch.randn(b["heads"], b["dim"], generator=g).to(torch.bfloat16)
            vec(q + "norm", n, 1.0); lin(q + "o", w, n)
        if L["mlp"]:
            ff = L["mlp"]["ff"]
            vec(f"l{i}.norm2", w)
            lin(f"l{i}.mlp.gate", ff, w, 1.3); lin(f"l{i}.mlp.up", ff, w, 1.3); lin(f"l{i}.mlp.down", w, ff)
    lin("head", cfg["vocab"], w)
    return W


MIXERS = {
    "latent": lat(3, 16, 8, 24, 32, 20), "latent of many heads": lat(20, 8, 8, 8, 136, 16), "latent of odd sizes": lat(1, 10, 6, 12, 9, 5), "latent on the matrix cores": lat(2, 96, 32, 64, 296, 72),
    "pair": par((4, 2, 16, 24, 8, 11, 3), (2, 16)), "pair of odd sizes": par((3, 1, 10, 7, 6, 5, 0), (3, 7), conv=3, rank=5), "one tap, wide heads": par((2, 2, 40, 16, 40, 20, 4), (1, 80), conv=1, rank=16),
    "left alone": par((2, 1, 32, 16, 16, 9, 2), (2, 16), rs=0.0), "right alone": par((2, 1, 32, 16, 16, 9, 2), (2, 16), ls=0.0), "negative": par((2, 1, 32, 16, 16, 9, 2), (2, 16), ls=-1.0, rs=0.25),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MIXERS))
def test_mixer_prompts_and_decoding(gpu, dtype, name):
    """A mixer as the model builds it, over scattered pages and slots that held something else."""
    width, lens, first = 48, [90, 7, 33], [70, 3, 32]
    L, W, mx, cache = mixer_case(gpu, dtype, MIXERS[name], width, len(name), page=8)
    g = torch.Generator().manual_seed(7)
    hs = [torch.randn(l, width, generator=g).to(dtype) for l in lens]
    want = [mo.mixer(npy(h), W, "l0.mix.", L, 1e-5) for h in hs]
    s0 = cache.alloc(); cache.begin_step([(s0, [0] * 50)]); s1 = cache.alloc(); cache.begin_step([(s1, [0] * 9)]); cache.release(s0)
    for t in cache.layers[0].values():
        if t.is_floating_point(): t.fill_(float("nan"))
    slots = [cache.alloc() for _ in lens]
    done, nxt = [0] * len(lens), list(first)
    while any(b > a for a, b in zip(done, nxt)):
        live = [i for i in range(len(lens)) if nxt[i] > done[i]]
        sb = cache.begin_step([(slots[i], [0] * (nxt[i] - done[i])) for i in live])
        y = mx.forward(torch.cat([hs[i][done[i]: nxt[i]] for i in live]).to(gpu), sb, cache.layers[0])
        for r, i in enumerate(live):
            at = sum(nxt[j] - done[j] for j in live[:r])
            a, b = y[at: at + nxt[i] - done[i]], want[i][done[i]: nxt[i]]
            scale = np.abs(want[i]).max()
            assert np.abs(npy(a) - b).max() < TOL[dtype] * scale, (done, i)
        done, nxt = nxt, [min(x + 1, l) for x, l in zip(nxt, lens)]


# ---- whole models ------------------------------------------------------------------------------------------------------------------------------

MODELS = {
    # both mixers, layers without a feed-forward, layers that use another's weights -- one of them through another that does
    "mixed": dict(layers=[par((4, 2, 16, 24, 8, 11, 3), (2, 16), 40), lat(3, 16, 8, 24, 32, 20, 56), par((2, 2, 24, 16, 24, 30, 1), (3, 8), None, conv=2), {"weights_of": 1}, {"weights_of": 0},
                          lat(2, 24, 8, 16, 40, 16, None), {"weights_of": 3}], width=64, eps=1e-5),
    # sizes that no vector access fits, one key/value head, nothing kept, a window of one
    "odd": dict(layers=[par((3, 1, 10, 7, 6, 1, 0), (3, 7), 33, conv=3, rank=5), lat(1, 10, 6, 12, 9, 5, 21), par((2, 1, 6, 5, 2, 4, 2), (1, 11), 19, conv=1, rank=3)], width=36, eps=1e-3),
    # the sizes of the matrix-core kernels, more kept tokens than the window is long
    "matrix": dict(layers=[lat(4, 32, 16, 32, 64, 48, 96), par((4, 1, 64, 48, 32, 40, 70), (2, 64), 64, rank=16), lat(20, 16, 16, 16, 136, 24, 64)], width=128, eps=1e-6),
    # one pair alone, heads of time mixing too wide for the fused norm
    "wide": dict(layers=[par((2, 2, 32, 32, 32, 64, 4), (2, 80), 128, rank=24)], width=96, eps=1e-6),
}


def config(name):
    d = MODELS[name]
    layers = []
    for L in d["layers"]:
        if "weights_of" in L:
            L = dict(layers[L["weights_of"]], weights_of=L["weights_of"])
        layers.append(L)
    return {"architecture": "Menerax", "vocab": VOCAB, "width": d["width"], "norm": {"eps": d["eps"]}, "layers": layers}


def save(folder, cfg, W):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(W, os.path.join(folder, "model.safetensors"))
    return str(folder)


@pytest.fixture(scope="module")
def zoo(gpu, tmp_path_factory):
    from exllamav3_amd.registry import load_model
    held = {}

    def get(name, dtype):
        if name not in held:
            cfg = config(name)
            W = weights(cfg, len(name))
            held[name] = (cfg, {k: npy(v) for k, v in W.items()}, save(tmp_path_factory.mktemp(name), cfg, W), {})
        cfg, W, folder, models = held[name]
        if dtype not in models:
            models[dtype] = load_model(folder, device=gpu, dtype=dtype)
        return cfg, W, models[dtype], folder
    return get


_truth = {}


def truth(name, cfg, W, toks, taps=None):
    key = (name, tuple(toks))
    if key not in _truth or taps is not None:
        _truth[key] = mo.forward(cfg, W, toks, taps)
    return _truth[key]


def tokens(n, seed):
    return torch.randint(0, VOCAB, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def check(got, want, dtype):
    got = npy(got) if isinstance(got, torch.Tensor) else got
    err = got - want
    err -= err.mean(-1, keepdims=True)
    e = np.sqrt((err ** 2).mean(-1)) / want.std()
    # norms on small sublayer outputs amplify rounding row by row: bfloat16 is held tightly in the median and loosely in the worst row
    assert e.max() < (3e-5 if dtype == torch.float32 else 2e-1) and np.median(e) < (1e-5 if dtype == torch.float32 else 4e-2), (float(e.max()), int(e.argmax()), float(np.median(e)))


def run(model, cache, reqs, prompts):
    """reqs: token lists in one batch, the first prompts[i] tokens as one step, then one token each per step until the longest ends; per request [T, vocab]."""
    slots = [cache.alloc() for _ in reqs]
    outs = [[] for _ in reqs]
    at = list(prompts)
    sb = cache.begin_step([(s, t[:p]) for s, t, p in zip(slots, reqs, prompts)], [list(range(p)) for p in prompts])
    lg = npy(model.step(sb, cache))
    k = 0
    for i, p in enumerate(prompts):
        outs[i].append(lg[k: k + p]); k += p
    live = list(range(len(reqs)))
    while True:
        for i in [i for i in live if at[i] == len(reqs[i])]:
            cache.release(slots[i]); live.remove(i)
        if not live:
            return [np.concatenate(o) for o in outs]
        lg = npy(model.step(cache.begin_step([(slots[i], [reqs[i][at[i]]]) for i in live]), cache))
        for r, i in enumerate(live):
            outs[i].append(lg[r: r + 1]); at[i] += 1


def poison(cache):
    """Everything a slot or page holds becomes NaN: a sequence may read only what it wrote itself."""
    for layer in cache.layers:
        for t in layer.values():
            if t.is_floating_point():
                t.fill_(float("nan"))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_whole_prompt_and_the_stream_after_every_layer(gpu, zoo, name, dtype):
    cfg, W, model, _ = zoo(name, dtype)
    for n in (1, 2, 31, 130):
        toks, taps = tokens(n, n), []
        want = truth(name, cfg, W, toks, taps)
        model.layer_taps = []
        cache = model.new_cache(); poison(cache)
        got = run(model, cache, [toks], [n])[0]
        assert len(model.layer_taps) == len(taps) == len(cfg["layers"])
        for i, (a, b) in enumerate(zip(model.layer_taps, taps)):
            e = np.sqrt(np.mean((npy(a) - b) ** 2) / np.mean(b ** 2))
            assert e < (1e-5 if dtype == torch.float32 else 6e-2), (n, i, float(e))
        model.layer_taps = None
        check(got, want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
@pytest.mark.parametrize("prompt", [1, 2, 40, 65])
def test_prompt_then_token_by_token(gpu, zoo, name, dtype, prompt):
    cfg, W, model, _ = zoo(name, dtype)
    toks = tokens(100, 7)
    cache = model.new_cache(slots=1); poison(cache)
    check(run(model, cache, [toks], [prompt])[0], truth(name, cfg, W, toks), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_unequal_batch_with_reused_slots_and_pages(gpu, zoo, name, dtype):
    cfg, W, model, _ = zoo(name, dtype)
    reqs = [tokens(n, 20 + n) for n in (3, 90, 34, 66, 1)]
    prompts = [1, 70, 33, 64, 1]
    cache = model.new_cache(slots=2)
    for turn in range(2):                                           # the second turn runs over what the first one left
        poison(cache)
        got = run(model, cache, reqs, prompts)
        for t, o in zip(reqs, got):
            check(o, truth(name, cfg, W, t), dtype)
        assert cache.in_use() == 0 and cache.pages_in_use() == 0
    if dtype == torch.float32:
        for t, p, o in zip(reqs, prompts, got):                      # and against each request alone
            assert rel(run(model, cache, [t], [p])[0], o) < 3e-5


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(gpu, zoo, dtype):
    cfg, W, model, _ = zoo("mixed", dtype)
    toks = tokens(420, 3)
    check(run(model, model.new_cache(slots=1), [toks], [5])[0], truth("mixed", cfg, W, toks), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["matrix", "wide"])
def test_long_prompt_in_parallel_segments(gpu, zoo, name, dtype):
    """Prompts long enough that time mixing runs in segments, next to one that has fewer of them."""
    cfg, W, model, _ = zoo(name, dtype)
    reqs = [tokens(600, 5), tokens(70, 6)]
    mix = next(b.mixer.right for b in model.blocks if hasattr(b.mixer, "right"))
    cache = model.new_cache()
    assert mix.segments(cache.begin_step([(cache.alloc(), reqs[0])])) is not None
    for t, o in zip(reqs, run(model, model.new_cache(), reqs, [590, 70])):
        check(o, truth(name, cfg, W, t), dtype)


def test_layers_that_share_weights_keep_states_of_their_own(gpu, zoo):
    _, _, model, _ = zoo("mixed", torch.float32)
    cache = model.new_cache()
    assert model.cfg.weights_of == [0, 1, 2, 1, 0, 5, 1] and model.blocks[6] is model.blocks[3] is model.blocks[1] and model.blocks[4] is model.blocks[0]
    for name, layers in (("latent", (1, 3, 5, 6)), ("S", (0, 2, 4)), ("ring_k", (0, 2, 4)), ("conv", (0, 2, 4)), ("last", (0, 2, 4))):
        assert len({cache.layers[i][name].data_ptr() for i in layers}) == len(layers)


def test_weights_of_the_joint_product_are_held_once(gpu, zoo):
    _, _, model, _ = zoo("mixed", torch.bfloat16)
    m = model.blocks[0].mixer
    assert m.left.w_o.data_ptr() == m.w_o.data_ptr() and m.right.w_o.untyped_storage().data_ptr() == m.w_o.untyped_storage().data_ptr()
    assert model.blocks[2].mlp is None and model.blocks[2].norm2 is None


def test_a_step_that_continues_by_several_tokens_is_refused(gpu, zoo):
    _, _, model, _ = zoo("mixed", torch.float32)
    cache = model.new_cache()
    s = cache.alloc()
    model.step(cache.begin_step([(s, [1, 2, 3])]), cache)
    with pytest.raises(RuntimeError, match="continues"):
        cache.begin_step([(s, [4, 5])])


def test_trace_replay(gpu, zoo, tmp_path):
    from exllamav3_amd.trace import TraceSession
    cfg, W, model, _ = zoo("mixed", torch.float32)
    a, b = tokens(12, 1), tokens(5, 2)
    lines = [{"step": 0, "entries": [{"id": "a", "tokens": a[:11], "want": [0, 10]}, {"id": "b", "tokens": b[:4], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[11:], "want": []}, {"id": "b", "tokens": b[4:], "want": [0]}], "end": ["a"]},
             {"step": 2, "entries": [], "end": ["b"]}]
    out = io.StringIO()
    ses = TraceSession(model, str(tmp_path), max_tokens=64)
    ses.run([json.dumps(l) for l in lines], out)
    assert out.getvalue() == "done 0\ndone 1\ndone 2\n" and ses.cache.in_use() == 0
    r0 = np.fromfile(tmp_path / "0.f32", "<f4").reshape(2, VOCAB); r1 = np.fromfile(tmp_path / "1.f32", "<f4").reshape(1, VOCAB)
    check(r0.astype(np.float64), truth("mixed", cfg, W, a)[[0, 10]], torch.float32)
    check(r1.astype(np.float64), truth("mixed", cfg, W, b)[[4]], torch.float32)
    assert not os.path.exists(tmp_path / "2.f32")


@pytest.mark.parametrize("name", list(MODELS))
def test_greedy_generation_through_the_scheduler(gpu, zoo, name):
    """Continuous batching (a batch cap below the number of jobs), decode steps replayed as graphs: every job equals the oracle's own greedy continuation."""
    from exllamav3_amd.generator import Generator
    cfg, W, model, _ = zoo(name, torch.float32)
    prompts = [tokens(n, 50 + n) for n in (3, 40, 1, 17)]
    gen = Generator(model, max_batch=3)
    outs = gen.generate(prompts, 8)
    assert gen.graph_replays > 0 and gen.cache.in_use() == 0
    for p, o in zip(prompts, outs):
        seq = list(p)
        for t in o:
            lg = mo.forward(cfg, W, seq)[-1]
            assert lg[t] > lg.max() - 1e-3
            seq.append(t)
    assert Generator(model, graphs=False, max_batch=2).generate(prompts, 8) == outs


@pytest.mark.parametrize("dtype", DTYPES)
def test_captured_decode_steps_equal_eager_ones_replay_after_replay(gpu, zoo, dtype):
    """The same jobs with and without graphs over many replays, other work between them."""
    from exllamav3_amd.generator import Generator
    _, _, model, _ = zoo("matrix", dtype)
    prompts = [tokens(n, 60 + n) for n in (30, 9)]
    a, b = Generator(model), Generator(model, graphs=False)
    outs = a.generate(prompts, 40)
    assert a.graph_replays >= 30 and outs == b.generate(prompts, 40)


def test_command_line_generates(gpu, zoo, capsys):
    from exllamav3_amd import cli
    from exllamav3_amd.generator import Generator
    _, _, model, folder = zoo("mixed", torch.float32)
    assert cli.main(["generate", "--model", folder, "--dtype", "float32", "--tokens", "1,2,3", "--max-new-tokens", "4"]) == 0
    line = [l for l in capsys.readouterr().out.splitlines() if l.startswith("{")][-1]
    assert json.loads(line)["output"] == Generator(model).generate([[1, 2, 3]], 4)[0]
