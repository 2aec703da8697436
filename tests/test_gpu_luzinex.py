"""GPU tests of the Luzinex design (csrc/mix_retention.hip, the paged part of mix_latent.hip, kept first tokens and element-wise gates in mix_attn*.hip and
mix_diffattn.hip, the two-norm residual update of mix_canon.hip, modules.py, luzinex.py) against the float64 oracle of tests/luzinex_oracle.py: every mechanism alone, whole
models of several small shapes (written to a checkpoint folder and loaded through the registry), prefill against token-by-token decoding, unequal batches against
each request alone, slots and pages that are freed and used again, one dominant key far back, at page borders and at every edge of a window, the first tokens, long
decoding, trace replay and greedy generation through the scheduler.  float32 runs are held to float32 rounding; bfloat16 runs to a loose bar (the oracle does not
round)."""
import io
import json
import math
import os
import numpy as np
import pytest
import torch
import luzinex_oracle as lo

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 3e-5, torch.bfloat16: 4e-2}


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


def rows_of(gpu, lens, pos0=None, slots=None):
    """cu, tok_seq, tok_pos, slots, pos0, len_after of a packed step."""
    pos0 = pos0 or [0] * len(lens)
    slots = slots or list(range(len(lens)))
    cu = [0]
    for l in lens: cu.append(cu[-1] + l)
    seq = [i for i, l in enumerate(lens) for _ in range(l)]
    pos = [pos0[i] + j for i, l in enumerate(lens) for j in range(l)]
    return mk(gpu, cu), mk(gpu, seq), mk(gpu, pos), mk(gpu, slots), mk(gpu, pos0), mk(gpu, [p + l for p, l in zip(pos0, lens)])


def freqs(gpu, dims, base):
    from exllamav3_amd.modules import rotary_frequencies
    return rotary_frequencies(dims, base)[0].to(gpu).contiguous() if dims else None


def powers(gpu, decay):
    from exllamav3_amd import mix_ops
    return (torch.tensor(decay, dtype=torch.float64)[:, None] ** torch.arange(mix_ops.RETENTION_TILE + 1, dtype=torch.float64)[None]).float().to(gpu).contiguous()


# ---- the mechanisms alone -----------------------------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [36, 72, 1032])
def test_residual_update_with_two_norms(gpu, dtype, width):
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(width)
    n = 5
    x, y = torch.randn(n, width, generator=g), torch.randn(n, width + 8, generator=g).to(dtype)[:, :width]
    w1, w2 = torch.rand(width, generator=g) + 0.5, torch.rand(width, generator=g) - 0.5
    for mode, base in ((mix_ops.RES_KEEP, npy(x)), (mix_ops.RES_ADD, npy(x) + npy(y)), (mix_ops.RES_SET, npy(y))):
        xd = x.to(gpu)
        h1 = torch.empty(n, width, dtype=dtype, device=gpu); h2 = torch.empty_like(h1)
        yd = None if mode == mix_ops.RES_KEEP else y.to(gpu)
        mix_ops.residual_norm_pair(xd, yd, mode, w1.to(gpu), h1, w2.to(gpu), h2, 1e-3)
        assert rel(xd, base) < 1e-6
        assert rel(h1, lo.rms_norm(base, npy(w1), 1e-3)) < TOL[dtype] / 4 and rel(h2, lo.rms_norm(base, npy(w2), 1e-3)) < TOL[dtype] / 4
    xd = x.to(gpu)
    mix_ops.residual_norm_pair(xd, y.to(gpu), mix_ops.RES_ADD, None, None, None, None, 1e-3)       # the bare update
    assert rel(xd, npy(x) + npy(y)) < 1e-6


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [40, 37])
def test_gated_gelu_into_a_column_block(gpu, dtype, ff):
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(ff)
    z = torch.randn(6, 2 * ff, generator=g).mul(3).to(dtype)
    wide = torch.full((6, ff + 24), 7.0, dtype=dtype, device=gpu)
    zd = z.to(gpu)
    mix_ops.glu_act(wide[:, 24:], zd[:, :ff], zd[:, ff:], mix_ops.GLU_GELU_TANH)
    want = lo.gelu_tanh(npy(z)[:, :ff]) * npy(z)[:, ff:]
    assert rel(wide[:, 24:], want) < TOL[dtype] / 4 and bool((wide[:, :24] == 7.0).all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("interleaved", [True, False])
@pytest.mark.parametrize("off,dims", [(0, 8), (6, 10), (12, 4)])
def test_rotation_of_a_part_of_every_head(gpu, dtype, interleaved, off, dims):
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(dims)
    H, step, pos = 3, 16, [0, 1, 5, 999, 4000]
    q = torch.randn(len(pos), H * step, generator=g).to(dtype)
    want = npy(q).reshape(len(pos), H, step)
    want[:, :, off: off + dims] = lo.rotate(want[:, :, off: off + dims], pos, dims, 10000.0, interleaved)
    qd = q.to(gpu)
    mix_ops.rotate_heads(qd, mk(gpu, pos), freqs(gpu, dims, 10000.0), 1.0, interleaved, H, step, off)
    assert rel(qd.reshape(len(pos), H, step), want) < (5e-4 if dtype == torch.float32 else 1e-2)      # float32 angles at position 4000


def attend_window(gpu, dtype, q, k, sink, gate, size, keep, dims, base, G, scale, lens, decode_from, slots, mfma=None):
    """Rotation, cache store and attention of the kept window for sequences of rows q [T, H, d], k [T, G, d] (values = keys before rotation): the first decode_from[i]
    rows as one packed prompt step, the rest token by token.  Returns per sequence [T, H * d]."""
    from exllamav3_amd import mix_ops
    H, d = q[0].shape[1:]
    rows = keep + size
    rk = torch.full((max(slots) + 2, rows, G, d), float("nan"), dtype=dtype, device=gpu); rv = rk.clone()
    freq = freqs(gpu, dims, base)
    outs = [[] for _ in lens]

    def step(lo_, hi_):
        ln = [b - a for a, b in zip(lo_, hi_)]
        live = [i for i, l in enumerate(ln) if l > 0]
        ln = [ln[i] for i in live]
        cu, seq, pos, sl, p0, la = rows_of(gpu, ln, [lo_[i] for i in live], [slots[i] for i in live])
        pick = lambda t: torch.cat([t[i][lo_[i]: hi_[i]].reshape(hi_[i] - lo_[i], -1) for i in live]).to(dtype)
        # the column blocks of one wide product, as a model has them
        wide = torch.cat([pick(q), pick(k), pick(gate)], dim=1).to(gpu)
        qv, kv, gv = wide[:, : H * d], wide[:, H * d: (H + G) * d], wide[:, (H + G) * d:]
        kr = torch.empty(wide.shape[0], G * d, dtype=dtype, device=gpu)
        mix_ops.qk_prep(qv, kv, kv, None, None, freq, 1.0, True, 0.0, rk, rv, seq, pos, sl, la, d, k_out=kr, keep_first=keep)
        assert torch.equal(kv.float().cpu(), pick(k).float())                                  # the values stay as projected
        wide_out = torch.full((wide.shape[0], H * d + 8), 3.0, dtype=dtype, device=gpu)
        out = wide_out[:, : H * d]
        if lo_[live[0]] == 0:
            mix_ops.attn_prefill_maps(out, qv, kr, kv, gv, sink.to(gpu), cu, seq, pos, H, G, 1, d, d, scale, 0.0, size, mix_ops.MASK_WINDOW, max_rows=max(ln), keep=keep, mfma=mfma)
        else:
            mix_ops.attn_decode_maps(out, qv, rk, rv, gv, sink.to(gpu), sl, la, H, 1, scale, 0.0, mix_ops.MASK_WINDOW)
        assert bool((wide_out[:, H * d:] == 3.0).all())
        at = 0
        for i, l in zip(live, ln):
            outs[i].append(npy(out[at: at + l])); at += l

    step([0] * len(lens), decode_from)
    done = list(decode_from)
    while any(a < l for a, l in zip(done, lens)):
        nxt = [min(a + 1, l) for a, l in zip(done, lens)]
        step(done, nxt); done = nxt
    return [np.concatenate(o) for o in outs]


def window_truth(q, k, sink, gate, size, keep, dims, base, G, scale, dtype):
    q, k, gate = (npy(t.to(dtype)) for t in (q, k, gate))
    T, H, d = q.shape
    qr, kr = lo.rotate(q, range(T), dims, base, True), lo.rotate(k, range(T), dims, base, True)
    see = lo.kept_window(size, keep)
    o = np.concatenate([lo.softmax_read(qr[:, h], kr[:, h // (H // G)], k[:, h // (H // G)], scale, see, float(sink[h])) for h in range(H)], axis=1)
    return o * lo.sigmoid(gate.reshape(T, -1))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dims,size,keep", [(4, 2, 16, 8, 9, 3), (2, 2, 24, 24, 33, 1), (3, 1, 10, 4, 5, 0), (6, 2, 64, 16, 70, 66), (1, 1, 8, 2, 1, 2), (2, 1, 72, 8, 64, 64)])
def test_kept_window_attention_prompts_and_decoding(gpu, dtype, H, G, d, dims, size, keep):
    g = torch.Generator().manual_seed(size + d)
    lens, first = [150, 41, keep + 2], [110, 37, keep + 1]
    q = [torch.randn(l, H, d, generator=g) for l in lens]; k = [torch.randn(l, G, d, generator=g) for l in lens]
    gate = [torch.randn(l, H, d, generator=g) for l in lens]
    sink = torch.randn(H, generator=g)
    scale = 1.3 / math.sqrt(d)
    got = attend_window(gpu, dtype, q, k, sink, gate, size, keep, dims, 5000.0, G, scale, lens, first, [2, 0, 1])
    for i in range(len(lens)):
        want = window_truth(q[i], k[i], sink, gate[i], size, keep, dims, 5000.0, G, scale, dtype)
        assert rel(got[i], want) < TOL[dtype], i


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("size,keep,T", [(40, 5, 300), (64, 64, 260), (1, 3, 90), (37, 0, 200)])
def test_one_key_stands_out_at_every_edge_of_the_window(gpu, dtype, decoded, size, keep, T):
    """Row i = T - 1 and one loud key at j: in sight it takes nearly all the weight, out of sight it must leave no trace."""
    d = 16
    i = T - 1
    for j in sorted({0, max(keep - 1, 0), keep, keep + 1, i - size - 1, i - size, i - size + 1, i - size + 2, i - 1, i, T // 2}):
        if not 0 <= j <= i:
            continue
        g = torch.Generator().manual_seed(j)
        q, k, gate = torch.randn(T, 1, d, generator=g), 0.1 * torch.randn(T, 1, d, generator=g), torch.randn(T, 1, d, generator=g)
        q[i, 0], k[j, 0] = 0.0, 0.0
        q[i, 0, d - 1], k[j, 0, d - 1] = 12.0, 9.0                     # outside the rotated part: the score does not depend on the distance
        sink = torch.tensor([0.5])
        first = T - 3 if decoded else T
        got = attend_window(gpu, dtype, [q], [k], sink, [gate], size, keep, 8, 5000.0, 1, 0.25, [T], [first], [0])[0]
        want = window_truth(q, k, sink, gate, size, keep, 8, 5000.0, 1, 0.25, dtype)
        assert rel(got[i], want[i]) < TOL[dtype], j
        seen = i - j < size or j < keep
        loud = np.abs(want[i] / lo.sigmoid(npy(gate)[i, 0]))[d - 1]
        assert (loud > 8.0) == seen, j


@pytest.mark.parametrize("d,dv", [(64, 64), (40, 72), (64, 200), (50, 30), (96, 64), (128, 128), (104, 248), (160, 48), (192, 128), (150, 130), (144, 200), (224, 64), (256, 128), (256, 256), (201, 77)])
@pytest.mark.parametrize("window,keep", [(1 << 30, 0), (45, 5), (200, 70)])
def test_prompt_attention_on_the_matrix_cores_at_every_head_size(gpu, d, dv, window, keep):
    """Every tiling of the kernel (key and value sizes, 16 or 32 rows per wave, aligned rows or not): two unequal sequences, a result in a column block, a gate per
    value element, and scores that grow and shrink along the keys by far more than the step at which the running maximum moves."""
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(d + dv)
    lens, H, G, bf = [275, 37], 2, 1, torch.bfloat16
    n = sum(lens)
    q, k, v, gate = (torch.randn(n, w, generator=g) for w in (H * d, G * d, G * dv, H * dv))
    ramp = torch.cat([torch.linspace(0.1, 3.0, 100), torch.linspace(3.0, 0.1, 100), torch.linspace(0.1, 6.0, n - 200)])[:, None]
    q, k, v, gate = q.to(bf), (k * ramp).to(bf), v.to(bf), gate.to(bf)
    sink, scale = torch.tensor([0.3, -2.0]), 1.0 / math.sqrt(d)
    pad = 8 if (dv % 4 == 0) else 3
    wide_out = torch.full((n, H * dv + pad), 5.0, dtype=bf, device=gpu)
    cu, seq, pos, sl, p0, la = rows_of(gpu, lens)
    mix_ops.attn_prefill_maps(wide_out[:, : H * dv], q.to(gpu), k.to(gpu), v.to(gpu), gate.to(gpu), sink.to(gpu), cu, seq, pos, H, G, 1, d, dv, scale, 0.0, window, mix_ops.MASK_WINDOW,
                              max_rows=max(lens), mfma=True, keep=keep)
    assert bool((wide_out[:, H * dv:] == 5.0).all())
    at = 0
    for l in lens:
        qn, kn, vn, gn = (npy(t[at: at + l]) for t in (q, k, v, gate))
        see = lo.kept_window(window, keep)
        want = np.concatenate([lo.softmax_read(qn.reshape(l, H, d)[:, h], kn, vn, scale, see, float(sink[h])) for h in range(H)], axis=1) * lo.sigmoid(gn)
        assert rel(wide_out[at: at + l, : H * dv], want) < 1.5e-2
        at += l


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_sink_that_takes_most_of_the_weight(gpu, dtype):
    g = torch.Generator().manual_seed(5)
    T, H, d = 70, 2, 16
    q, k, gate = (torch.randn(T, H, d, generator=g) for _ in range(3))
    outs = []
    for sink in (torch.tensor([6.0, -30.0]), torch.tensor([-30.0, 6.0])):
        got = attend_window(gpu, dtype, [q], [k], sink, [gate], 20, 2, 8, 5000.0, H, 0.25, [T], [60], [0])[0]
        assert rel(got, window_truth(q, k, sink, gate, 20, 2, 8, 5000.0, H, 0.25, dtype)) < TOL[dtype]
        outs.append(got.reshape(T, H, d))
    assert np.abs(outs[0][5:, 0]).max() < 0.5 * np.abs(outs[1][5:, 0]).max() and np.abs(outs[1][5:, 1]).max() < 0.5 * np.abs(outs[0][5:, 1]).max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,dv,dims,interleaved", [(2, 32, 48, 32, False), (3, 24, 20, 8, False), (1, 64, 64, 64, True), (2, 128, 72, 128, False), (1, 200, 33, 100, False), (1, 7, 5, 0, False)])
@pytest.mark.parametrize("segments", [None, (3, 64), (4, 32)])
def test_retention_prompt_then_decoding(gpu, dtype, H, d, dv, dims, interleaved, segments):
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(d)
    lens, extra = [125, 32, 1, 33], 4
    decay = [0.5, 0.97, 0.9995][:H]
    slots = [3, 1, 4, 0]
    q, k = ([torch.randn(l + extra, H * d, generator=g).to(dtype) for l in lens] for _ in range(2))
    v, gt = ([torch.randn(l + extra, H * dv, generator=g).to(dtype) for l in lens] for _ in range(2))
    state = torch.full((6, H, d, dv), float("nan"), device=gpu)
    pw, freq = powers(gpu, decay), freqs(gpu, dims, 7000.0)
    want, last = [], []
    for i, l in enumerate(lens):
        T = l + extra
        qr, kr = (lo.rotate(npy(t[i]).reshape(T, H, d), range(T), dims, 7000.0, interleaved) for t in (q, k))
        kr = kr * d ** -0.5
        o = [lo.retention_scan(qr[:, h], kr[:, h], npy(v[i]).reshape(T, H, dv)[:, h], decay[h]) for h in range(H)]
        want.append(np.stack([a for a, _ in o], axis=1)); last.append(np.stack([S for _, S in o]))
    wide = torch.cat([torch.cat([t[i][:l] for t in (q, k, v)], dim=1) for i, l in enumerate(lens)]).to(gpu)
    cols = lambda w: (w[:, : H * d], w[:, H * d: 2 * H * d], w[:, 2 * H * d: 2 * H * d + H * dv])
    cu, seq, pos, sl, p0, la = rows_of(gpu, lens, None, slots)
    o = torch.full((wide.shape[0], H, dv), float("nan"), device=gpu)
    mix_ops.retention(o, state, *cols(wide), pw, freq, interleaved, cu, sl, p0, d ** -0.5, segments=segments)
    at = 0
    for i, l in enumerate(lens):
        assert rel(o[at: at + l], want[i][:l]) < 3e-5, i                      # float32 in both modes: the inputs are what they are
        at += l
    assert torch.isnan(state[2]).all() and torch.isnan(state[5]).all()
    for t in range(extra):
        w1 = torch.stack([torch.cat([x[i][l + t] for x in (q, k, v, gt)]) for i, l in enumerate(lens)]).to(gpu)
        wide_out = torch.full((len(lens), H * dv + 8), 2.0, dtype=dtype, device=gpu)
        mix_ops.retention_step(wide_out[:, : H * dv], state, *cols(w1), w1[:, 2 * H * d + H * dv:], pw, freq, interleaved, mk(gpu, [l + t for l in lens]), sl, H, d ** -0.5, 1e-5)
        ref = np.stack([(lo.rms_unit(want[i][l + t], 1e-5) * lo.silu(npy(gt[i][l + t]).reshape(H, dv))).reshape(-1) for i, l in enumerate(lens)])
        assert rel(wide_out[:, : H * dv], ref) < TOL[dtype] / 4, t
        assert bool((wide_out[:, H * dv:] == 2.0).all())
    for i in range(len(lens)):
        assert rel(state[slots[i]], last[i]) < 3e-5


def test_retention_forgets_nothing_with_a_decay_of_one_and_everything_with_zero(gpu):
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(1)
    T, H, d, dv = 300, 2, 16, 16
    q, k, v = (torch.randn(T, H * d, generator=g) for _ in range(3))
    cu, seq, pos, sl, p0, la = rows_of(gpu, [T])
    for seg in (None, (4, 96)):
        o = torch.empty(T, H, dv, device=gpu); state = torch.full((1, H, d, dv), float("nan"), device=gpu)
        mix_ops.retention(o, state, q.to(gpu), k.to(gpu), v.to(gpu), powers(gpu, [1.0, 0.0]), None, False, cu, sl, p0, 1.0, segments=seg)
        Q, K, V = (npy(t).reshape(T, H, d) for t in (q, k, v))
        assert rel(o[:, 0], lo.retention_scan(Q[:, 0], K[:, 0], V[:, 0], 1.0)[0]) < 3e-5
        assert rel(o[:, 1], (Q[:, 1] * K[:, 1]).sum(-1, keepdims=True) * V[:, 1]) < 3e-5


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("weightless", [True, False])
def test_head_norm_with_and_without_a_weight(gpu, dtype, weightless):
    from exllamav3_amd import mix_ops
    g = torch.Generator().manual_seed(3)
    n, H, dv = 4, 3, 20
    o, gt, w = torch.randn(n, H, dv, generator=g), torch.randn(n, H * dv, generator=g).to(dtype), torch.rand(dv, generator=g) + 0.5
    out = torch.empty(n, H * dv + 4, dtype=dtype, device=gpu)[:, : H * dv]
    mix_ops.head_norm_gate(out, o.to(gpu), None if weightless else w.to(gpu), gt.to(gpu), mix_ops.GATE_SILU, 1e-4)
    want = (lo.rms_unit(npy(o), 1e-4) * (1.0 if weightless else npy(w))).reshape(n, -1) * lo.silu(npy(gt))
    assert rel(out, want) < TOL[dtype] / 4


def latent_case(gpu, dtype, H, d, r, dv, rank, q_rank, width, T, page, seed):
    """A PagedLatentAttention (and a second one that reads its rows) with random weights against the oracle; the cache they share."""
    from exllamav3_amd.modules import PagedLatentAttention
    from exllamav3_amd.state_cache import SlotStateCache
    g = torch.Generator().manual_seed(seed)
    m = {"heads": H, "dim": d, "rot_dim": r, "vdim": dv, "kv_rank": rank, "q_rank": q_rank, "scale": 1.0 / math.sqrt(d + r), "rot": {"base": 20000.0, "dims": r}}
    lin = lambda o, i, s=1.0: (s * torch.randn(o, i, generator=g) / math.sqrt(i)).to(torch.bfloat16).float()
    W = {"a.dq": lin(q_rank, width), "a.dq.norm": torch.rand(q_rank, generator=g) + 0.5, "a.uq": lin(H * (d + r), q_rank, 2.0), "a.dkv": lin(rank + r, width),
         "a.dkv.norm": torch.rand(rank, generator=g) + 0.5, "a.uk": lin(H * d, rank), "a.uv": lin(H * dv, rank), "a.g": lin(H * dv, width), "a.o": lin(width, H * dv)}
    W.update({"b." + nm: lin(*W["a." + nm].shape, 1.5) for nm in ("dq", "uq", "uk", "uv", "g", "o")})
    W["b.dq.norm"] = torch.rand(q_rank, generator=g) + 0.5

    class Tensors:
        def get_tensor(self, key, device="cpu"):
            return W[key]
    lender = PagedLatentAttention(width, H, d, r, dv, rank, q_rank, m["scale"], 1e-6, r, 20000.0, gate=True, layer=0)
    reader = PagedLatentAttention(width, H, d, r, dv, rank, q_rank, m["scale"], 1e-6, r, 20000.0, gate=True, layer=1, kv_from=0)
    lender.load(Tensors(), "a.", dtype, gpu); reader.load(Tensors(), "b.", dtype, gpu)
    cache = SlotStateCache([lender.state_specs(), reader.state_specs()], gpu, slots=4, page_size=page)
    return m, {k: npy(v) for k, v in W.items()}, lender, reader, cache, g


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,r,dv,rank,q_rank,page", [(3, 16, 8, 24, 32, 20, 8), (2, 24, 16, 16, 40, 48, 64), (20, 8, 8, 8, 136, 16, 16), (1, 10, 6, 12, 9, 5, 4), (2, 96, 32, 64, 300, 72, 32)])
def test_paged_latent_attention_and_a_layer_that_reads_its_rows(gpu, dtype, H, d, r, dv, rank, q_rank, page):
    width, lens, first = 40, [90, 7, 33], [70, 3, 32]
    m, W, lender, reader, cache, g = latent_case(gpu, dtype, H, d, r, dv, rank, q_rank, width, max(lens), page, H + rank)
    hs = [torch.randn(l, width, generator=g).to(dtype) for l in lens]
    want = []
    for h in hs:
        c, kr = lo.latent_keys(npy(h), W, "a.", m, 1e-6)
        want.append((lo.latent_attention(npy(h), W, "a.", m, 1e-6, c, kr), lo.latent_attention(npy(h), W, "b.", m, 1e-6, c, kr)))
    # scattered pages: a sequence that grows and ends first leaves the free list in another order
    s0 = cache.alloc(); cache.begin_step([(s0, [0] * 50)]); s1 = cache.alloc(); cache.begin_step([(s1, [0] * 9)]); cache.release(s0)
    for t in cache.layers[0].values():
        if t.is_floating_point(): t.fill_(float("nan"))
    slots = [cache.alloc() for _ in lens]
    done, nxt = [0] * len(lens), list(first)
    while any(b > a for a, b in zip(done, nxt)):
        live = [i for i in range(len(lens)) if nxt[i] > done[i]]
        sb = cache.begin_step([(slots[i], [0] * (nxt[i] - done[i])) for i in live])
        h = torch.cat([hs[i][done[i]: nxt[i]] for i in live]).to(gpu)
        a = lender.forward(h, sb, cache.layers[0])
        b = reader.forward(h, sb, cache.layers[0])
        assert rel(a, np.concatenate([want[i][0][done[i]: nxt[i]] for i in live])) < TOL[dtype], done
        assert rel(b, np.concatenate([want[i][1][done[i]: nxt[i]] for i in live])) < TOL[dtype], done
        done, nxt = nxt, [min(x + 1, l) for x, l in zip(nxt, lens)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("decoded", [False, True])
def test_one_cached_row_stands_out_anywhere_behind_a_row(gpu, dtype, decoded):
    """Hundreds of cached rows, one of which takes nearly all of the last row's weight: first, last, at page borders, in the middle."""
    H, d, r, dv, rank, q_rank, page, width, T = 2, 16, 8, 16, 32, 24, 64, 48, 700
    m, W, lender, reader, cache, g = latent_case(gpu, dtype, H, d, r, dv, rank, q_rank, width, T, page, 9)
    base = torch.randn(T, width, generator=g)
    for j in (0, 1, 63, 64, 65, 127, 128, 350, 511, 512, 639, 640, T - 2, T - 1):
        h = base.clone()
        # key j offers what the row asks for: h_j is moved so that its unrotated key lies along the row's query (least squares through the latent)
        cq = lo.rms_norm(npy(h[T - 1:]) @ W["a.dq"].T, W["a.dq.norm"], 1e-6)
        qv = (cq @ W["a.uq"].T).reshape(H, d + r)[0, :d]
        target = W["a.uk"].reshape(H, d, rank)[0].T @ qv                       # latent direction that scores highest
        if j < T - 1:
            z = np.concatenate([target * W["a.dkv.norm"] * 40.0, np.zeros(r)])     # the latent that scores highest after its norm, no rotated part
            h[j] = torch.from_numpy(np.linalg.pinv(W["a.dkv"]) @ z).float()
        h = h.to(dtype)
        mm = dict(m, scale=m["scale"] * 6.0)
        c, kr = lo.latent_keys(npy(h), W, "a.", mm, 1e-6)
        # the oracle for the last row alone: rows before it only provide keys
        cq = lo.rms_norm(npy(h[T - 1:]) @ W["a.dq"].T, W["a.dq.norm"], 1e-6)
        q = (cq @ W["a.uq"].T).reshape(1, H, d + r)
        qr = lo.rotate(q[:, :, d:], [T - 1], r, m["rot"]["base"], False)
        heads, top = [], []
        for hd in range(H):
            s = (c @ W["a.uk"].reshape(H, d, rank)[hd].T @ q[0, hd, :d] + kr @ qr[0, hd]) * mm["scale"]
            p = np.exp(s - s.max()); p /= p.sum()
            top.append((int(p.argmax()), float(p.max())))
            heads.append(p @ (c @ W["a.uv"].reshape(H, dv, rank)[hd].T))
        want = (np.concatenate(heads) * lo.sigmoid(npy(h[T - 1]) @ W["a.g"].T)) @ W["a.o"].T
        if j < T - 1:
            assert top[0][0] == j and top[0][1] > 0.5, (j, top)
        lender.scale = mm["scale"]
        s = cache.alloc()
        k = T - 1 if decoded else T
        out = lender.forward(h[:k].to(gpu), cache.begin_step([(s, [0] * k)]), cache.layers[0])
        if decoded:
            out = lender.forward(h[k:].to(gpu), cache.begin_step([(s, [0])]), cache.layers[0])
        cache.release(s)
        assert rel(out[-1], want) < TOL[dtype] * (2 if dtype == torch.bfloat16 else 1), j


# ---- whole models ------------------------------------------------------------------------------------------------------------------------------

def lat(heads, dim, rot, vdim, rank, q_rank, ff=None, base=30000.0, **kw):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank, "scale": 1.5 / math.sqrt(dim + rot), "rot": {"base": base, "dims": rot}}
    m.update(kw)
    return {"type": "latent_attention", "mixer": m, "mlp": ff and {"kind": "dense", "ff": ff}}


def win(heads, kv, dim, dims, size, keep, ff=None, base=9000.0):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": 1.2 / math.sqrt(dim), "mask": {"size": size, "keep_first": keep},
                                           "rot": {"base": base, "dims": dims}}, "mlp": ff and {"kind": "dense", "ff": ff}}


def ret(dim, vdim, decay, dims, ff=None, base=40000.0):
    return {"type": "retention", "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": decay, "rot": {"base": base, "dims": dims}}, "mlp": ff and {"kind": "dense", "ff": ff}}


MODELS = {
    # every mechanism, a latent that two later layers read, layers without a feed-forward
    "mixed": dict(layers=[ret(16, 24, [0.9, 0.99], 8, 48), lat(3, 16, 8, 24, 32, 20, 40), win(4, 2, 16, 8, 11, 3, 56), lat(2, 24, 8, 16, 32, 16, None, kv_from=1), ret(24, 16, [0.97], 24, None),
                          lat(3, 16, 8, 24, 32, 24, 24, kv_from=1)], width=64, eps=1e-5),
    # sizes that no vector access fits, one key/value head, nothing kept, a window of one
    "odd": dict(layers=[win(3, 1, 10, 6, 7, 0, 33), lat(1, 10, 6, 12, 9, 5, 21), ret(7, 5, [0.8, 1.0, 0.999], 6, 19), win(2, 2, 6, 2, 1, 2, None)], width=36, eps=1e-3),
    # the attention layers alone at the sizes of the matrix-core kernels, two latents
    "latents": dict(layers=[lat(4, 32, 16, 32, 64, 48, 96), win(4, 4, 32, 32, 40, 70, 64), lat(20, 16, 16, 16, 136, 24, 64), lat(4, 48, 16, 40, 64, 40, 64, kv_from=0)], width=96, eps=1e-6),
    # retention alone, a single layer of it
    "retention": dict(layers=[ret(64, 64, [0.5, 0.98, 0.9995], 64, 128)], width=128, eps=1e-6),
}


def config(name):
    d = MODELS[name]
    return {"architecture": "Luzinex", "vocab": 91, "width": d["width"], "norm": {"eps": d["eps"]}, "layers": d["layers"]}


def weights(cfg, seed):
    g = torch.Generator().manual_seed(seed)
    w = cfg["width"]
    W = {}

    def lin(name, o, i, s=1.0):
        W[name] = (s * torch.randn(o, i, generator=g) / math.sqrt(i)).to(torch.bfloat16)

    def norm(name, n):
        W[name] = (0.6 + 0.8 * torch.rand(n, generator=g)).to(torch.bfloat16)
    W["embed"] = torch.randn(cfg["vocab"], w, generator=g).to(torch.bfloat16)
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], f"l{i}.mix."
        norm(f"l{i}.norm1", w)
        H = m["heads"]
        if L["type"] == "latent_attention":
            d, r, dv, rank = m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            lin(p + "dq", m["q_rank"], w); norm(p + "dq.norm", m["q_rank"]); lin(p + "uq", H * (d + r), m["q_rank"], 1.5)
            if "kv_from" not in m:
                lin(p + "dkv", rank + r, w, 1.5); norm(p + "dkv.norm", rank)
            lin(p + "uk", H * d, rank); lin(p + "uv", H * dv, rank); lin(p + "g", H * dv, w); lin(p + "o", w, H * dv)
        elif L["type"] == "attention":
            d = m["dim"]
            lin(p + "q", H * d, w, 1.5); lin(p + "k", m["kv_heads"] * d, w, 1.5); lin(p + "g", H * d, w); lin(p + "o", w, H * d)
            W[p + "sink"] = torch.randn(H, generator=g).to(torch.bfloat16)
        else:
            for nm, n in (("q", H * m["dim"]), ("k", H * m["dim"]), ("v", H * m["vdim"]), ("g", H * m["vdim"])):
                lin(p + nm, n, w)
            lin(p + "o", w, H * m["vdim"])
        if L["mlp"]:
            ff = L["mlp"]["ff"]
            norm(f"l{i}.norm2", w)
            lin(f"l{i}.mlp.gate", ff, w); lin(f"l{i}.mlp.up", ff, w); lin(f"l{i}.mlp.down", w, ff)
    norm("final.norm", w)
    lin("head", cfg["vocab"], w)
    return W


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
        _truth[key] = lo.forward(cfg, W, toks, taps)
    return _truth[key]


def tokens(n, seed):
    return torch.randint(0, 91, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def check(got, want, dtype):
    got = npy(got) if isinstance(got, torch.Tensor) else got
    err = got - want
    err -= err.mean(-1, keepdims=True)
    e = np.sqrt((err ** 2).mean(-1)) / want.std()
    assert e.max() < (2e-5 if dtype == torch.float32 else 8e-2), (float(e.max()), int(e.argmax()))


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
        assert len(model.layer_taps) == len(taps)
        for i, (a, b) in enumerate(zip(model.layer_taps, taps)):
            assert rel(a, b) < (2e-5 if dtype == torch.float32 else 5e-2), (n, i)
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
            assert rel(run(model, cache, [t], [p])[0], o) < 2e-5


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(gpu, zoo, dtype):
    cfg, W, model, _ = zoo("mixed", dtype)
    toks = tokens(420, 3)
    check(run(model, model.new_cache(slots=1), [toks], [5])[0], truth("mixed", cfg, W, toks), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_prompt_in_parallel_segments(gpu, zoo, dtype):
    """Prompts long enough that retention runs in segments, next to one that has fewer of them."""
    cfg, W, model, _ = zoo("retention", dtype)
    reqs = [tokens(600, 5), tokens(70, 6)]
    seg = model.blocks[0].mixer
    sb = model.new_cache()
    s = sb.alloc()
    assert seg.segments(sb.begin_step([(s, reqs[0])])) is not None
    for t, o in zip(reqs, run(model, model.new_cache(), reqs, [590, 70])):
        check(o, truth("retention", cfg, W, t), dtype)


def test_a_layer_reads_the_rows_of_another(gpu, zoo):
    """The pages exist once per lender; a borrowing layer brings none, and changing the lender's latent changes what it computes."""
    cfg, W, model, _ = zoo("mixed", torch.float32)
    cache = model.new_cache()
    assert "latent" in cache.layers[1] and not cache.layers[3] and not cache.layers[5] and model.cfg.source == [0, 1, 2, 1, 4, 1]


def test_weights_of_a_joint_product_are_held_once(gpu, zoo):
    _, _, model, _ = zoo("mixed", torch.bfloat16)
    b = model.blocks[0]
    assert b.mixer.w_o.data_ptr() == b.w_out.data_ptr() and b.mlp.w_down.untyped_storage().data_ptr() == b.w_out.untyped_storage().data_ptr()
    assert model.blocks[4].mlp is None and model.blocks[4].norm2 is None


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
    r0 = np.fromfile(tmp_path / "0.f32", "<f4").reshape(2, 91); r1 = np.fromfile(tmp_path / "1.f32", "<f4").reshape(1, 91)
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
            lg = lo.forward(cfg, W, seq)[-1]
            assert lg[t] > lg.max() - 1e-3
            seq.append(t)
    assert Generator(model, graphs=False, max_batch=2).generate(prompts, 8) == outs


def test_command_line_generates(gpu, zoo, capsys):
    from exllamav3_amd import cli
    from exllamav3_amd.generator import Generator
    _, _, model, folder = zoo("mixed", torch.float32)
    assert cli.main(["generate", "--model", folder, "--dtype", "float32", "--tokens", "1,2,3", "--max-new-tokens", "4"]) == 0
    line = [l for l in capsys.readouterr().out.splitlines() if l.startswith("{")][-1]
    assert json.loads(line)["output"] == Generator(model).generate([[1, 2, 3]], 4)[0]
