"""CPU tests around the Menerax design: closed forms that pin the float64 oracle (tests/menerax_oracle.py) independently of any kernel, mistakes planted in the oracle's
configuration that the GPU tests' inputs would show, the configuration reader, loading a written checkpoint without a GPU, the tile form of time mixing, blended rotary
frequencies, the registry and the C ABI's declarations."""
import json
import math
import numpy as np
import pytest
import torch
import menerax_oracle as mo


def test_oracle_norms():
    x = np.array([[3.0, 4.0]])
    assert np.allclose(mo.rms_norm(x, np.array([1.0, 2.0]), 0.0), np.array([[3.0, 8.0]]) / math.sqrt(12.5))
    assert np.allclose(mo.norm_around_zero(x, np.array([0.0, 1.0]), 0.0), np.array([[3.0, 8.0]]) / math.sqrt(12.5))          # the weight is a deviation from one
    assert np.allclose(mo.rms_unit(np.array([1.0, 1.0]), 3.0), 0.5)                                                         # eps inside the root


def test_oracle_rotation_pairs():
    x = np.arange(1.0, 7.0)[None]
    rot = {"dims": 4, "base": 100.0}
    a0, a1 = 3.0, 3.0 * 100.0 ** -0.5
    h = mo.rotate(x, [3], rot, False)[0]                                                             # pairs (0, 2) and (1, 3); entries 4, 5 stay
    assert np.allclose(h, [1 * math.cos(a0) - 3 * math.sin(a0), 2 * math.cos(a1) - 4 * math.sin(a1), 3 * math.cos(a0) + 1 * math.sin(a0), 4 * math.cos(a1) + 2 * math.sin(a1), 5, 6])
    i = mo.rotate(x, [3], rot, True)[0]                                                              # pairs (0, 1) and (2, 3)
    assert np.allclose(i, [1 * math.cos(a0) - 2 * math.sin(a0), 2 * math.cos(a0) + 1 * math.sin(a0), 3 * math.cos(a1) - 4 * math.sin(a1), 4 * math.cos(a1) + 3 * math.sin(a1), 5, 6])


def test_blended_frequencies_keep_the_fast_slow_the_slow_and_join_between():
    """By turns over the original context: pairs above `high` turns are kept, pairs below `low` get 1 / factor, and the blend meets both ends."""
    sc = {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 2048}
    for dims, base in ((64, 500000.0), (16, 10000.0), (6, 300.0)):
        plain = mo.pair_frequencies({"dims": dims, "base": base})
        scaled = mo.pair_frequencies({"dims": dims, "base": base, "scaling": sc})
        kinds = set()
        for f, s in zip(plain, scaled):
            turns = sc["original"] * f / (2 * math.pi)
            if turns > 4.0: assert s == f; kinds.add("kept")
            elif turns < 1.0: assert abs(s - f / 8) < 1e-15; kinds.add("slowed")
            else:
                share = (turns - 1.0) / 3.0
                assert abs(s - (share * f + (1 - share) * f / 8)) < 1e-12; kinds.add("blended")
        assert dims < 64 or kinds == {"kept", "slowed", "blended"}
        from exllamav3_amd.modules import rotary_frequencies
        got, mag = rotary_frequencies(dims, base, sc)
        assert mag == 1.0 and np.allclose(got.double().numpy(), scaled, rtol=1e-7) and np.allclose(rotary_frequencies(dims, base)[0].double().numpy(), plain, rtol=1e-7)


def test_other_scalings_are_untouched():
    from exllamav3_amd.modules import rotary_frequencies
    f, mag = rotary_frequencies(8, 10000.0, {"factor": 4.0, "original": 1024, "fast": 32, "slow": 1})
    assert abs(mag - (0.1 * math.log(4.0) + 1.0)) < 1e-12 and f.numel() == 4


def test_oracle_softmax_with_a_cap_and_the_kept_window():
    see = mo.kept_window(3, 2)
    assert [[j for j in range(8) if see(i, j)] for i in (0, 3, 4, 7)] == [[0], [0, 1, 2, 3], [0, 1, 2, 3, 4], [0, 1, 5, 6, 7]]
    q, k, v = np.array([[2.0], [2.0]]), np.array([[1.0], [3.0]]), np.array([[10.0], [20.0]])
    s = 5.0 * np.tanh(np.array([2.0, 6.0]) * 0.5 / 5.0)
    p = np.exp(s) / np.exp(s).sum()
    assert np.allclose(mo.softmax_read(q, k, v, 0.5, lambda i, j: j <= i, 5.0)[1], p @ v)


def test_oracle_short_convolution_and_token_shift():
    u, w = np.arange(1.0, 6.0)[:, None], np.array([[100.0, 10.0, 1.0]])
    assert np.allclose(mo.short_convolution(u, w)[:, 0], [1, 12, 123, 234, 345])                    # the last tap is the row's own, zeros ahead of the start
    assert np.allclose(mo.shifted_mix(u, np.array([0.25]))[:, 0], [0.75, 1.75, 2.75, 3.75, 4.75])     # h + (h' - h) mu, h' = 0 at the start
    assert np.allclose(mo.shifted_mix(u, np.array([1.0]))[:, 0], [0, 1, 2, 3, 4])


def test_oracle_time_mixing_against_its_sum():
    """o_t = sum_(j < t) (r_t . (prod_(j < s < t) w_s) k_j) v_j + (r_t . u k_t) v_t: a token's own decay does not act on its own write, the bonus only on the current one."""
    rng = np.random.default_rng(3)
    T, d, dv = 7, 3, 2
    r, k, v, w, u = rng.normal(size=(T, d)), rng.normal(size=(T, d)), rng.normal(size=(T, dv)), rng.uniform(0.2, 1.0, size=(T, d)), rng.normal(size=d)
    got, S = mo.time_mix_scan(r, k, v, w, u)
    for t in range(T):
        o = (r[t] * u * k[t]).sum() * v[t]
        for j in range(t):
            o = o + (r[t] * np.prod(w[j + 1: t], axis=0) * k[j]).sum() * v[j]
        assert np.allclose(got[t], o)
    assert np.allclose(S, sum(np.outer(np.prod(w[j + 1:], axis=0) * k[j], v[j]) for j in range(T)))
    assert np.allclose(mo.decay_of(np.array([-50.0, 0.0, 5.0])), [1.0, math.exp(-1), 0.0], atol=1e-20)


@pytest.mark.parametrize("strength", [0.05, 1.0, 9.0])
def test_time_mixing_in_tiles_equals_the_token_loop(strength):
    """What the prompt kernel computes, in float32 where it does: exponents counted from the middle of a tile of 16, strong tiles token by token, segments with a walk over
    them between two passes."""
    rng = np.random.default_rng(1)
    T, d, dv, tile = 75, 6, 5, 16
    r, k, v, u = rng.normal(size=(T, d)), rng.normal(size=(T, d)), rng.normal(size=(T, dv)), rng.normal(size=d)
    lw = -strength * rng.exponential(size=(T, d)) / math.log(2)                                       # base-2 logarithms
    want, last = mo.time_mix_scan(r, k, v, 2.0 ** lw, u)
    f = np.float32
    used = set()

    def tiles(a, b, S):
        out, total = [], np.zeros(d)
        for n0 in range(a, b, tile):
            n1 = min(n0 + tile, b)
            l = np.zeros((tile, d)); l[: n1 - n0] = lw[n0:n1]
            M, L15 = l[:8].sum(0), l.sum(0)
            total += L15
            if (M < -80).any() or (L15 - M < -80).any():
                used.add("loop")
                o, S1 = np.zeros((n1 - n0, dv)), S.copy()
                for t in range(n0, n1):
                    o[t - n0] = (S1 + u[:, None] * np.outer(k[t], v[t])).T @ r[t]
                    S1 = (2.0 ** lw[t])[:, None] * S1 + np.outer(k[t], v[t])
                S = S1
            else:
                used.add("tile")
                L = np.cumsum(l, axis=0)
                q = r[n0:n1].astype(f) * (2.0 ** (L - l - M))[: n1 - n0].astype(f)
                p = k[n0:n1].astype(f) * (2.0 ** (M - L))[: n1 - n0].astype(f)
                A = np.tril(q @ p.T, -1) + np.diag((r[n0:n1] * u * k[n0:n1]).sum(1)).astype(f)
                Sm = (2.0 ** M)[:, None] * S
                o = q @ Sm.astype(f) + A @ v[n0:n1].astype(f)
                S = (2.0 ** (L15 - M))[:, None] * (Sm + p.T @ v[n0:n1].astype(f))
            out.append(o)
        return np.concatenate(out), S, total
    scale = np.abs(want).max()
    o, S, _ = tiles(0, T, np.zeros((d, dv)))
    assert np.abs(o - want).max() < 1e-5 * scale and np.abs(S - last).max() < 1e-5 * np.abs(last).max()
    S, seg = np.zeros((d, dv)), 32
    for s in range(0, T, seg):                                                                        # local contributions, then the state each segment starts from
        e = min(s + seg, T)
        assert np.abs(tiles(s, e, S)[0] - want[s:e]).max() < 1e-5 * scale
        _, local, total = tiles(s, e, np.zeros((d, dv)))
        S = (2.0 ** total)[:, None] * S + local
    assert np.abs(S - last).max() < 1e-5 * np.abs(last).max()
    assert used == ({"tile"} if strength < 5 else {"loop"} if used == {"loop"} else {"tile", "loop"})


LAYERS = [{"type": "latent_attention", "mixer": {"heads": 2, "dim": 6, "rot_dim": 4, "vdim": 5, "kv_rank": 8, "q_rank": 7, "scale": 0.3, "rot": {"base": 100.0, "dims": 4}}, "mlp": None},
          {"type": "parallel", "mixer": {"left": {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 3, "conv": 3, "scale": 0.4, "softcap": 4.0, "mask": {"size": 5, "keep_first": 2},
                                                  "rot": {"base": 200.0, "dims": 4, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 200}}},
                                         "right": {"heads": 2, "dim": 4}, "left_scale": 0.75, "right_scale": 1.5}, "mlp": {"kind": "dense", "ff": 12, "limit": 0.5}}]
LAYERS = LAYERS + [dict(LAYERS[1], weights_of=1), dict(LAYERS[0], weights_of=0)]
BASE = {"architecture": "Menerax", "vocab": 11, "width": 16, "norm": {"eps": 1e-4}, "layers": LAYERS}


def _weights(cfg, g):
    w, W = cfg["width"], {}
    rnd = lambda *s: 0.5 * torch.randn(*s, generator=g)
    W["embed"], W["head"], W["embed.norm"], W["final.norm"] = rnd(cfg["vocab"], w), rnd(cfg["vocab"], w), torch.full((w,), 0.25), torch.full((w,), -0.25)
    for i, L in enumerate(cfg["layers"]):
        if "weights_of" in L:
            continue
        m, p = L["mixer"], f"l{i}.mix."
        W[f"l{i}.norm1"] = torch.full((w,), 0.125)
        if L["type"] == "latent_attention":
            H, d, r, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            W[p + "dq"], W[p + "dq.norm"], W[p + "uq"] = rnd(m["q_rank"], w), torch.ones(m["q_rank"]), rnd(H * (d + r), m["q_rank"])
            W[p + "dkv"], W[p + "dkv.norm"], W[p + "uk"], W[p + "uv"] = rnd(rank + r, w), torch.ones(rank), rnd(H * d, rank), rnd(H * dv, rank)
            W[p + "g"], W[p + "o"] = rnd(H, w), rnd(w, H * dv)
        else:
            a, b = m["left"], m["right"]
            for nm, n in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
                W[p + f"left.{nm}"], W[p + f"left.{nm}.b"], W[p + f"left.{nm}.conv"] = rnd(n, w), rnd(n), rnd(n, a["conv"])
            W[p + "left.q.norm"], W[p + "left.k.norm"] = torch.full((a["dim"],), 1.5), torch.full((a["dim"],), 0.75)
            W[p + "left.g"], W[p + "left.o"] = rnd(a["heads"] * a["vdim"], w), rnd(w, a["heads"] * a["vdim"])
            q, n = p + "right.", b["heads"] * b["dim"]
            for nm in "rkvg":
                W[q + nm] = rnd(n, w)
            for nm in "rkvgw":
                W[q + "mu." + nm] = torch.rand(w, generator=g)
            W[q + "w1"], W[q + "w2"], W[q + "w0"], W[q + "u"], W[q + "norm"], W[q + "o"] = rnd(5, w), rnd(n, 5), rnd(n) - 1, rnd(b["heads"], b["dim"]), torch.ones(n), rnd(w, n)
        if L["mlp"]:
            ff = L["mlp"]["ff"]
            W[f"l{i}.norm2"] = torch.full((w,), 0.5)
            W[f"l{i}.mlp.gate"], W[f"l{i}.mlp.up"], W[f"l{i}.mlp.down"] = rnd(ff, w), rnd(ff, w), rnd(w, ff)
    return W


def test_oracle_norms_sit_on_the_sublayers_outputs():
    cfg = dict(BASE, layers=[LAYERS[1]])
    W = {k.replace("l1.", "l0."): v.double().numpy() for k, v in _weights(BASE, torch.Generator().manual_seed(3)).items() if not k.startswith("l0.")}
    taps, toks = [], [1, 5, 2]
    lg = mo.forward(cfg, W, toks, taps)
    x = mo.norm_around_zero(W["embed"][toks], W["embed.norm"], 1e-4)
    x = x + mo.norm_around_zero(mo.mixer(x, W, "l0.mix.", LAYERS[1], 1e-4), W["l0.norm1"], 1e-4)
    x = x + mo.norm_around_zero(mo.feed_forward(x, W, "l0.mlp.", 0.5), W["l0.norm2"], 1e-4)
    assert np.allclose(taps[0], x) and np.allclose(lg, mo.norm_around_zero(x, W["final.norm"], 1e-4) @ W["head"].T)


def test_planted_mistakes_show():
    """Each mistake in a copy of the configuration moves the oracle's logits: the models' inputs see every constant."""
    W = {k: v.double().numpy() for k, v in _weights(BASE, torch.Generator().manual_seed(4)).items()}
    toks = [1, 2, 3, 4, 5, 6, 7, 8, 9, 10, 0, 3]
    want = mo.forward(BASE, W, toks)
    for i, path, value in ((0, ("mixer", "scale"), 0.31), (0, ("mixer", "rot", "base"), 110.0), (1, ("mixer", "left", "mask", "size"), 6), (1, ("mixer", "left", "mask", "keep_first"), 1),
                           (1, ("mixer", "left", "rot", "dims"), 6), (1, ("mixer", "left", "rot", "base"), 210.0), (1, ("mixer", "left", "rot", "scaling", "factor"), 5.0),
                           (1, ("mixer", "left", "rot", "scaling", "original"), 150), (1, ("mixer", "left", "rot", "scaling", "high"), 6.0), (1, ("mixer", "left", "softcap"), 4.2),
                           (1, ("mixer", "left", "scale"), 0.41), (1, ("mixer", "left_scale"), 0.76), (1, ("mixer", "right_scale"), 1.45), (1, ("mlp", "limit"), 0.55)):
        cfg = json.loads(json.dumps(BASE))
        d = cfg["layers"][i]
        for key in path[:-1]:
            d = d[key]
        d[path[-1]] = value
        assert np.abs(mo.forward(cfg, W, toks) - want).max() > 1e-4, (i, path)


def _broken(change):
    cfg = json.loads(json.dumps(BASE))
    change(cfg["layers"])
    return cfg


@pytest.mark.parametrize("change,text", [
    (lambda L: L[2].update(weights_of=9), "weights_of 9"),
    (lambda L: L[1].update(weights_of=2), "weights_of 1"),                                           # 1 -> 2 -> 1
    (lambda L: L[2].update(weights_of=0), "describes another layer"),
    (lambda L: L[2]["mixer"].update(left_scale=0.7), "describes another layer"),
    (lambda L: (L.pop(), L[1].update(type="window"), L.pop()), "unknown mixer"),
    (lambda L: (L.pop(), L.pop(), L[1]["mlp"].update(kind="moe")), "unknown feed-forward"),
    (lambda L: (L.pop(), L.pop(), L[1]["mixer"]["left"].update(kv_heads=3)), "over 3 key/value heads"),
    (lambda L: (L.pop(), L.pop(), L[1]["mixer"]["left"]["rot"].update(dims=8)), "8 rotated dimensions of 6"),
    (lambda L: (L.pop(), L.pop(), L[1]["mixer"]["left"].update(conv=17)), "17 taps"),
    (lambda L: (L.pop(), L.pop(), L[1]["mixer"]["right"].update(dim=300)), "at most 256"),
    (lambda L: L.clear(), "no layers")])
def test_configurations_that_do_not_fit_are_refused(change, text):
    from exllamav3_amd.menerax import MeneraxConfig
    with pytest.raises(RuntimeError, match=text):
        MeneraxConfig(_broken(change)).build_blocks()


def test_model_from_a_written_checkpoint_on_the_cpu(tmp_path):
    """Loading needs no GPU: tensors land where the mechanisms expect them, and layers that share weights are one block with states of their own."""
    from safetensors.torch import save_file
    from exllamav3_amd import registry
    W = _weights(BASE, torch.Generator().manual_seed(0))
    with open(tmp_path / "config.json", "w") as f:
        json.dump(BASE, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in W.items()}, str(tmp_path / "model.safetensors"))
    m = registry.load_model(str(tmp_path), "cpu", torch.float32)
    assert m.architecture == "Menerax" and m.vocab == 11 and len(m.blocks) == 4 and m.cfg.weights_of == [0, 1, 1, 0] and m.blocks[2] is m.blocks[1] and m.blocks[3] is m.blocks[0]
    a, b = m.blocks[:2]
    assert a.mixer.inp.weight.shape == (7 + 12 + 2, 16) and a.mixer.interleaved and a.norm2 is None and a.mlp is None and torch.equal(a.norm1, torch.full((16,), 1.125))
    left, right = b.mixer.left, b.mixer.right
    assert left.inp.weight.shape == (24 + 12 + 6 + 12, 16) and left.inp.bias is not None and bool((left.inp.bias[42:] == 0).all()) and not left.interleaved and left.sink is None
    conv = torch.cat([W[f"l1.mix.left.{nm}.conv"] for nm in "qkv"]).to(torch.bfloat16).float()
    assert torch.equal(left.conv, conv.t()) and left.softcap == 4.0 and left.out_scale == 0.75
    assert torch.equal(right.norm_w, torch.full((8,), 1.5)) and right.w_in.shape == (4 * 8 + 5, 16) and torch.equal(right.w_mix[2], W["l1.mix.right.v"].to(torch.bfloat16).float())
    joint = torch.cat([W["l1.mix.left.o"], W["l1.mix.right.o"]], dim=1).to(torch.bfloat16).float()
    assert torch.equal(b.mixer.w_o, joint) and left.w_o.data_ptr() == b.mixer.w_o.data_ptr() and torch.equal(right.w_o, joint[:, 12:]) and b.mlp.limit == 0.5
    assert torch.equal(m.embed_norm, torch.full((16,), 1.25)) and torch.equal(m.final_norm, torch.full((16,), 0.75))
    cache = m.new_cache(slots=3, tokens=100)
    assert set(cache.layers[0]) == {"latent", "page_table"} == set(cache.layers[3]) and set(cache.layers[1]) == {"ring_k", "ring_v", "conv", "S", "last"} == set(cache.layers[2])
    assert cache.layers[1]["ring_k"].shape == (3, 7, 2, 6) and cache.layers[1]["ring_v"].shape == (3, 7, 2, 3) and cache.layers[1]["conv"].shape == (3, 2, 42)
    assert cache.layers[1]["S"].shape == (3, 2, 4, 4) and cache.layers[1]["last"].shape == (3, 16) and cache.layers[1]["S"].data_ptr() != cache.layers[2]["S"].data_ptr()


def test_mixers_side_by_side_need_states_of_different_names():
    from exllamav3_amd.modules import SummedMixers, TimeMix
    with pytest.raises(RuntimeError, match="same name"):
        SummedMixers(16, TimeMix(16, 2, 4, 1e-5), TimeMix(16, 1, 8, 1e-5)).state_specs()


def test_segments_cover_the_longest_prompt():
    from exllamav3_amd import mix_ops
    from exllamav3_amd.modules import TimeMix
    from exllamav3_amd.state_cache import StepBatch
    for heads, dim in ((1, 64), (4, 64), (16, 128), (64, 64), (96, 256)):
        t = TimeMix(64, heads, dim, 1e-5)
        for rows in (1, 255, 256, 300, 1000, 4096, 100000):
            for batch in (1, 7):
                s = t.segments(StepBatch(n=rows, batch=batch, decode=False, max_rows=rows, tokens=None, cu=None, tok_seq=None, tok_pos=None, slots=None, pos0=None, len_after=None))
                if s is not None:
                    assert s[0] >= 1 and s[0] * s[1] >= rows and (s[0] - 1) * s[1] < rows and s[1] % mix_ops.TIMEMIX_TILE == 0 and rows >= 256


def test_products_off_the_gpu_or_of_many_rows_are_vendor_products():
    from exllamav3_amd import mix_ops
    from exllamav3_amd.modules import linear
    x, w, b = torch.randn(3, 16).to(torch.bfloat16), torch.randn(5, 16).to(torch.bfloat16), torch.randn(5).to(torch.bfloat16)
    assert not mix_ops.skinny_ok(x, w) and torch.equal(linear(x, w, b), torch.nn.functional.linear(x, w, b))


def test_registered_and_declared():
    from exllamav3_amd import _lib, registry
    assert "Menerax" in registry.architectures() and registry.native_libraries("Menerax") == ("mix",)
    names = _lib.mix_declared_symbols()
    for n in ("exl3_mix_embed_norm", "exl3_mix_conv_prep", "exl3_mix_token_shift", "exl3_mix_decay_log2", "exl3_mix_timemix", "exl3_mix_timemix_step", "exl3_mix_skinny"):
        assert n in names
    assert _lib.check_mix_symbols()
