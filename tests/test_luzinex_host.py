"""CPU tests around the Luzinex design: closed forms that pin the float64 oracle (tests/luzinex_oracle.py) independently of any kernel, mistakes planted in the oracle
that the GPU tests' inputs would show, the configuration reader, loading a written checkpoint without a GPU, the tile form of retention, where a window with kept
first tokens puts a position, the registry and the C ABI's declarations."""
import json
import math
import numpy as np
import pytest
import torch
import luzinex_oracle as lo


def test_oracle_norm_and_activation():
    assert np.allclose(lo.rms_norm(np.array([[3.0, 4.0]]), np.array([1.0, 2.0]), 0.0), np.array([[3.0, 8.0]]) / math.sqrt(12.5))
    assert np.allclose(lo.rms_unit(np.array([1.0, 1.0]), 3.0), 0.5)                                  # eps inside the root
    z = np.linspace(-4, 4, 9)
    assert np.allclose(lo.gelu_tanh(z), torch.nn.functional.gelu(torch.from_numpy(z), approximate="tanh").numpy(), atol=1e-12)


def test_oracle_rotation_pairs_and_partial():
    x = np.arange(1.0, 7.0)[None]
    a0, a1 = 3.0, 3.0 * 100.0 ** -0.5
    h = lo.rotate(x, [3], 4, 100.0, False)[0]                                                        # pairs (0, 2) and (1, 3); entries 4, 5 stay
    assert np.allclose(h, [1 * math.cos(a0) - 3 * math.sin(a0), 2 * math.cos(a1) - 4 * math.sin(a1), 3 * math.cos(a0) + 1 * math.sin(a0), 4 * math.cos(a1) + 2 * math.sin(a1), 5, 6])
    i = lo.rotate(x, [3], 4, 100.0, True)[0]                                                         # pairs (0, 1) and (2, 3)
    assert np.allclose(i, [1 * math.cos(a0) - 2 * math.sin(a0), 2 * math.cos(a0) + 1 * math.sin(a0), 3 * math.cos(a1) - 4 * math.sin(a1), 4 * math.cos(a1) + 3 * math.sin(a1), 5, 6])
    assert np.allclose(lo.rotate(x, [0], 6, 100.0, True), x)


def test_oracle_softmax_with_a_sink_and_the_kept_window():
    see = lo.kept_window(3, 2)
    assert [[j for j in range(8) if see(i, j)] for i in (0, 3, 4, 7)] == [[0], [0, 1, 2, 3], [0, 1, 2, 3, 4], [0, 1, 5, 6, 7]]
    assert [j for j in range(8) if lo.kept_window(1, 0)(7, j)] == [7]
    q, k, v = np.zeros((3, 2)), np.zeros((3, 2)), np.array([[3.0], [6.0], [9.0]])
    assert np.allclose(lo.softmax_read(q, k, v, 1.0, lambda i, j: j <= i)[:, 0], [3.0, 4.5, 6.0])
    assert np.allclose(lo.softmax_read(q, k, v, 1.0, lambda i, j: j <= i, sink=math.log(2.0))[:, 0], [1.0, 9.0 / 4, 18.0 / 5])      # two more shares of nothing


def test_oracle_latent_attention_equals_the_absorbed_form():
    """Scores through per-head keys equal scores of the absorbed query against the cached latent: what a decode step computes."""
    rng = np.random.default_rng(0)
    w, H, d, r, dv, rank, qr, T = 10, 2, 4, 2, 3, 5, 6, 7
    m = {"heads": H, "dim": d, "rot_dim": r, "vdim": dv, "kv_rank": rank, "q_rank": qr, "scale": 0.4, "rot": {"base": 50.0, "dims": r}}
    W = {"m." + nm: rng.normal(size=s) for nm, s in (("dq", (qr, w)), ("dq.norm", (qr,)), ("uq", (H * (d + r), qr)), ("dkv", (rank + r, w)), ("dkv.norm", (rank,)), ("uk", (H * d, rank)),
                                                     ("uv", (H * dv, rank)), ("g", (H * dv, w)))}
    W["m.o"] = np.eye(H * dv)
    h = rng.normal(size=(T, w))
    c, kr = lo.latent_keys(h, W, "m.", m, 1e-5)
    got = lo.latent_attention(h, W, "m.", m, 1e-5, c, kr)
    cq = lo.rms_norm(h @ W["m.dq"].T, W["m.dq.norm"], 1e-5)
    q = (cq @ W["m.uq"].T).reshape(T, H, d + r)
    qrot = lo.rotate(q[:, :, d:], range(T), r, 50.0, False)
    t, hd = T - 1, 1
    ql = W["m.uk"].reshape(H, d, rank)[hd].T @ q[t, hd, :d]
    s = (c @ ql + kr @ qrot[t, hd]) * 0.4
    p = np.exp(s) / np.exp(s).sum()
    want = (W["m.uv"].reshape(H, dv, rank)[hd] @ (p @ c)) * lo.sigmoid(h[t] @ W["m.g"].T)[hd * dv:]
    assert np.allclose(got[t, hd * dv:], want)


def test_retention_in_tiles_equals_the_token_loop():
    """What the prompt kernel computes, with its own split into tiles and segments: O = diag(g^(t+1)) Q S + (Q K^T . D) V, S <- g^T S + (diag(g^(T-1-t)) K)^T V."""
    rng = np.random.default_rng(1)
    T, d, dv, g = 45, 6, 5, 0.93
    q, k, v = rng.normal(size=(T, d)), rng.normal(size=(T, d)), rng.normal(size=(T, dv))
    want, last = lo.retention_scan(q, k, v, g)

    def tiles(lo_, hi_, S, size):
        out = []
        for n0 in range(lo_, hi_, size):
            n1 = min(n0 + size, hi_)
            t = np.arange(n1 - n0)
            D = np.where(t[:, None] >= t[None], g ** np.maximum(t[:, None] - t[None], 0), 0.0)
            out.append((g ** (t + 1))[:, None] * (q[n0:n1] @ S) + ((q[n0:n1] @ k[n0:n1].T) * D) @ v[n0:n1])
            S = g ** len(t) * S + ((g ** (len(t) - 1 - t))[:, None] * k[n0:n1]).T @ v[n0:n1]
        return np.concatenate(out), S
    for size in (1, 4, 16, 64):
        o, S = tiles(0, T, np.zeros((d, dv)), size)
        assert np.allclose(o, want) and np.allclose(S, last)
    S, seg = np.zeros((d, dv)), 20
    for s in range(0, T, seg):                                                                        # local contributions, then the state each segment starts from
        e = min(s + seg, T)
        assert np.allclose(tiles(s, e, S, 16)[0], want[s:e])
        S = g ** (e - s) * S + tiles(s, e, np.zeros((d, dv)), 16)[1]
    assert np.allclose(S, last)


def ring_entry(pos, rows, keep):
    return pos if pos < keep else keep + (pos - keep) % (rows - keep)


def ring_holds(pos, length, rows, keep):
    return pos < keep or pos >= length - (rows - keep)


@pytest.mark.parametrize("size,keep", [(5, 3), (1, 2), (4, 0), (7, 7)])
def test_a_slot_of_kept_and_recent_rows_holds_exactly_what_is_visible(size, keep):
    """The placement rule of the cache kernels: after any split into a prompt and decoded rows, the first min(len, keep + size) entries are the visible positions."""
    rows = keep + size
    see = lo.kept_window(size, keep)
    for prompt in range(1, 30):
        held = {}
        for p in range(prompt):
            if ring_holds(p, prompt, rows, keep):
                assert ring_entry(p, rows, keep) not in held
                held[ring_entry(p, rows, keep)] = p
        for length in range(prompt, 31):
            if length > prompt:
                p = length - 1
                assert ring_holds(p, length, rows, keep)
                held[ring_entry(p, rows, keep)] = p
            assert [held[e] for e in range(min(length, rows))] and sorted(held[e] for e in range(min(length, rows))) == [j for j in range(length) if see(length - 1, j)]


LAYERS = [{"type": "latent_attention", "mixer": {"heads": 2, "dim": 6, "rot_dim": 4, "vdim": 5, "kv_rank": 8, "q_rank": 7, "scale": 0.3, "rot": {"base": 100.0, "dims": 4}}, "mlp": None},
          {"type": "attention", "mixer": {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 6, "scale": 0.4, "mask": {"size": 5, "keep_first": 2}, "rot": {"base": 200.0, "dims": 2}},
           "mlp": {"kind": "dense", "ff": 12}},
          {"type": "retention", "mixer": {"heads": 2, "dim": 4, "vdim": 3, "decay": [0.5, 0.9], "rot": {"base": 300.0, "dims": 4}}, "mlp": {"kind": "dense", "ff": 10}},
          {"type": "latent_attention", "mixer": {"heads": 3, "dim": 2, "rot_dim": 4, "vdim": 5, "kv_rank": 8, "q_rank": 9, "scale": 0.3, "kv_from": 0, "rot": {"base": 100.0, "dims": 4}},
           "mlp": {"kind": "dense", "ff": 9}}]
BASE = {"architecture": "Luzinex", "vocab": 11, "width": 16, "norm": {"eps": 1e-4}, "layers": LAYERS}


def _weights(cfg, g):
    w, W = cfg["width"], {}
    rnd = lambda *s: 0.5 * torch.randn(*s, generator=g)
    W["embed"], W["head"], W["final.norm"] = rnd(cfg["vocab"], w), rnd(cfg["vocab"], w), torch.full((w,), 0.75)
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], f"l{i}.mix."
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        W[f"l{i}.norm1"] = torch.full((w,), 1.25)
        if L["type"] == "latent_attention":
            W[p + "dq"], W[p + "dq.norm"], W[p + "uq"] = rnd(m["q_rank"], w), torch.ones(m["q_rank"]), rnd(H * (d + m["rot_dim"]), m["q_rank"])
            W[p + "uk"], W[p + "uv"] = rnd(H * d, m["kv_rank"]), rnd(H * dv, m["kv_rank"])
            if "kv_from" not in m:
                W[p + "dkv"], W[p + "dkv.norm"] = rnd(m["kv_rank"] + m["rot_dim"], w), torch.ones(m["kv_rank"])
        elif L["type"] == "attention":
            W[p + "q"], W[p + "k"], W[p + "sink"] = rnd(H * d, w), rnd(m["kv_heads"] * d, w), rnd(H)
        else:
            W[p + "q"], W[p + "k"], W[p + "v"] = rnd(H * d, w), rnd(H * d, w), rnd(H * dv, w)
        W[p + "g"], W[p + "o"] = rnd(H * dv, w), rnd(w, H * dv)
        if L["mlp"]:
            ff = L["mlp"]["ff"]
            W[f"l{i}.norm2"] = torch.full((w,), 0.5)
            W[f"l{i}.mlp.gate"], W[f"l{i}.mlp.up"], W[f"l{i}.mlp.down"] = rnd(ff, w), rnd(ff, w), rnd(w, ff)
    return W


def test_oracle_runs_both_norms_of_the_same_stream_in_parallel():
    cfg = dict(BASE, layers=[LAYERS[2]])
    W = {k: v.double().numpy() for k, v in _weights(cfg, torch.Generator().manual_seed(3)).items()}
    taps, toks = [], [1, 5, 2]
    lg = lo.forward(cfg, W, toks, taps)
    x = W["embed"][toks]
    y = lo.retention(lo.rms_norm(x, W["l0.norm1"], 1e-4), W, "l0.mix.", LAYERS[2]["mixer"], 1e-4) + lo.feed_forward(lo.rms_norm(x, W["l0.norm2"], 1e-4), W, "l0.mlp.")
    assert np.allclose(taps[0], x + y) and np.allclose(lg, lo.rms_norm(x + y, W["final.norm"], 1e-4) @ W["head"].T)


def test_planted_mistakes_show():
    """Each mistake in a copy of the configuration moves the oracle's logits: the models' inputs see every constant."""
    W = {k: v.double().numpy() for k, v in _weights(BASE, torch.Generator().manual_seed(4)).items()}
    toks = [1, 2, 3, 4, 5, 6, 7, 8, 9, 10, 0, 3]
    want = lo.forward(BASE, W, toks)
    for i, path, value in ((0, ("scale",), 0.31), (0, ("rot", "base"), 110.0), (1, ("mask", "size"), 6), (1, ("mask", "keep_first"), 1), (1, ("rot", "dims"), 4), (2, ("decay",), [0.5, 0.89]),
                           (2, ("rot", "base"), 310.0), (2, ("rot", "dims"), 2), (3, ("rot", "base"), 90.0)):
        cfg = json.loads(json.dumps(BASE))
        d = cfg["layers"][i]["mixer"]
        for key in path[:-1]:
            d = d[key]
        d[path[-1]] = value
        assert np.abs(lo.forward(cfg, W, toks) - want).max() > 1e-4, (i, path)


def _broken(change):
    cfg = json.loads(json.dumps(BASE))
    change(cfg["layers"])
    return cfg


@pytest.mark.parametrize("change,text", [
    (lambda L: L[3]["mixer"].update(kv_from=1), "latent of layer 1"),
    (lambda L: L[3]["mixer"].update(kv_from=3 + 4), "latent of layer 7"),
    (lambda L: L[3]["mixer"].update(kv_rank=9), "rank or rotation"),
    (lambda L: L[3]["mixer"]["rot"].update(base=101.0), "rank or rotation"),
    (lambda L: L.append(json.loads(json.dumps(dict(L[3], mixer=dict(L[3]["mixer"], kv_from=3))))), "latent of layer 3"),
    (lambda L: L[1].update(type="window"), "unknown mixer"),
    (lambda L: L[1]["mlp"].update(kind="moe"), "unknown feed-forward"),
    (lambda L: L[1]["mixer"].update(kv_heads=3), "over 3 key/value heads"),
    (lambda L: L[1]["mixer"].update(vdim=5), "have their size"),
    (lambda L: L[2]["mixer"].update(decay=[0.5]), "1 decays for 2 heads"),
    (lambda L: L.clear(), "no layers")])
def test_configurations_that_do_not_fit_are_refused(change, text):
    from exllamav3_amd.luzinex import LuzinexConfig
    with pytest.raises(RuntimeError, match=text):
        LuzinexConfig(_broken(change)).build_blocks()


def test_model_from_a_written_checkpoint_on_the_cpu(tmp_path):
    """Loading needs no GPU: tensors land where the mechanisms expect them, and a layer that reads another's rows is given that layer's state."""
    from safetensors.torch import save_file
    from exllamav3_amd import registry
    W = _weights(BASE, torch.Generator().manual_seed(0))
    with open(tmp_path / "config.json", "w") as f:
        json.dump(BASE, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in W.items()}, str(tmp_path / "model.safetensors"))
    m = registry.load_model(str(tmp_path), "cpu", torch.float32)
    assert m.architecture == "Luzinex" and m.vocab == 11 and len(m.blocks) == 4 and m.cfg.source == [0, 1, 2, 0]
    a, b, c, d = m.blocks
    assert a.mixer.inp.weight.shape == (7 + 12 + 10, 16) and d.mixer.inp.weight.shape == (9 + 15, 16) and a.norm2 is None and a.mlp is None
    assert a.mixer.w_uk_padded.shape == (2 * 10, 8) and bool((a.mixer.w_uk_padded.view(2, 10, 8)[:, 6:] == 0).all()) and a.mixer.w_uv_heads_t.is_contiguous()
    assert b.mixer.inp.weight.shape == (24 + 12 + 24, 16) and b.mixer.tied and b.mixer.sink.dtype == torch.float32
    joint = torch.cat([W["l1.mix.o"], W["l1.mlp.down"]], dim=1).to(torch.bfloat16).float()
    assert torch.equal(b.w_out, joint) and b.mixer.w_o.data_ptr() == b.w_out.data_ptr() and torch.equal(b.mlp.w_down, joint[:, 24:])
    assert torch.equal(c.mixer.pw[:, :3], torch.tensor([[1.0, 0.5, 0.25], [1.0, 0.9, 0.81]], dtype=torch.float64).float()) and abs(float(c.mixer.freq[1]) - 300.0 ** -0.5) < 1e-7
    cache = m.new_cache(slots=3, tokens=100)
    assert set(cache.layers[0]) == {"latent", "page_table"} and set(cache.layers[1]) == {"ring_k", "ring_v"} and set(cache.layers[2]) == {"S"} and not cache.layers[3]
    assert cache.layers[0]["latent"].shape[1:] == (m.PAGE_SIZE, 12) and cache.layers[1]["ring_k"].shape == (3, 7, 2, 6) and cache.layers[2]["S"].shape == (3, 2, 4, 3)


def test_segments_cover_the_longest_prompt():
    from exllamav3_amd import mix_ops
    from exllamav3_amd.modules import Retention
    from exllamav3_amd.state_cache import StepBatch
    for heads, vdim in ((1, 64), (4, 64), (16, 128), (64, 256)):
        r = Retention(64, heads, 64, vdim, [0.9] * heads, 0, 1.0, 1e-5)
        for rows in (1, 255, 256, 300, 1000, 4096, 100000):
            for batch in (1, 7):
                sb = StepBatch(n=rows, batch=batch, decode=False, max_rows=rows, tokens=None, cu=None, tok_seq=None, tok_pos=None, slots=None, pos0=None, len_after=None)
                s = r.segments(sb)
                if s is not None:
                    assert s[0] >= 1 and s[0] * s[1] >= rows and (s[0] - 1) * s[1] < rows and s[1] % mix_ops.RETENTION_TILE == 0 and rows >= 256


def test_registered_and_declared():
    from exllamav3_amd import _lib, registry
    assert "Luzinex" in registry.architectures() and registry.native_libraries("Luzinex") == ("mix",)
    names = _lib.mix_declared_symbols()
    for n in ("exl3_mix_residual_norm_pair", "exl3_mix_latent_rows", "exl3_mix_rotate_heads", "exl3_mix_retention", "exl3_mix_retention_step"):
        assert n in names
    assert _lib.check_mix_symbols()
