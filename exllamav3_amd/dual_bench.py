"""
`bench.py --dual-family`: prefill and decode throughput of Luzinex layers (parallel blocks with two norms: paged latent attention, kept-window attention or
retention beside a gated gelu feed-forward; random weights) at sizes that resemble real models' layers, beside the closest existing models of the same library,
timed in the same process at the same width and head shapes and with feed-forwards of (nearly) the same weight count -- Zagilorn's latent attention (a window
as long as the prompt, so that it reads the same keys), Vofanex's window attention and its gated linear attention -- and each kernel of the design alone against
its roofline, next to the like kernel of those models.  Prints one JSON line; the default workload of bench.py and the JSON line it prints are untouched.
"""
from __future__ import annotations
import json
import math
import time
import torch
from . import latent_bench
from .latent_bench import LATENT
from .mixer_bench import PEAK_BF16, PEAK_F32, PEAK_HBM, SIZES, TensorDict, _time, kernel_legs, model_legs

KINDS = [("latent_attention", "dense"), ("attention", "dense"), ("retention", "dense")]
Q_RANK, KEEP_FIRST = 1536, 4


def gated_ff(size: dict) -> int:
    """Three matrices where the compared layers have two: two thirds of their width."""
    return -(-size["ff"] * 2 // (3 * 128)) * 128


def synth(size: dict, lt: dict, kinds, vocab=32000, seed=0, device="cuda:0", share=False):
    """Random Luzinex weights and their config: size as in mixer_bench.SIZES, lt as in latent_bench.LATENT (q_rank: Q_RANK if it has none).  share: every
    second latent layer reads the rows of the one before it."""
    g = torch.Generator(device=device).manual_seed(seed)
    w, t, layers, ff = size["width"], {}, [], gated_ff(size)
    q_rank, lender = lt.get("q_rank", Q_RANK), None

    def lin(name, o, i, s=1.0):
        t[name] = (torch.randn(o, i, generator=g, device=device) * (s / math.sqrt(i))).to(torch.bfloat16)

    def vec(name, n, mean=0.0, s=0.1):
        t[name] = (mean + s * torch.randn(n, generator=g, device=device)).to(torch.bfloat16)
    lin("embed", vocab, w, math.sqrt(w)); lin("head", vocab, w); vec("final.norm", w, 1.0)
    for i, (mix, mlp) in enumerate(kinds):
        p = f"l{i}.mix."
        vec(f"l{i}.norm1", w, 1.0)
        if mix == "latent_attention":
            H, d, r, dv, rank = lt["heads"], lt["dim"], lt["rot_dim"], lt["vdim"], lt["rank"]
            lin(p + "dq", q_rank, w); vec(p + "dq.norm", q_rank, 1.0); lin(p + "uq", H * (d + r), q_rank)
            lin(p + "uk", H * d, rank); lin(p + "uv", H * dv, rank)
            mixer = {"heads": H, "dim": d, "rot_dim": r, "vdim": dv, "kv_rank": rank, "q_rank": q_rank, "scale": (d + r) ** -0.5, "rot": {"base": 10000.0, "dims": r}}
            if share and lender is not None:
                mixer["kv_from"], lender = lender, None
            else:
                lin(p + "dkv", rank + r, w); vec(p + "dkv.norm", rank, 1.0)
                lender = i
        elif mix == "attention":
            H, G, d = size["heads"], size["kv_heads"], size["dim"]
            dv = d
            lin(p + "q", H * d, w); lin(p + "k", G * d, w); vec(p + "sink", H)
            mixer = {"heads": H, "kv_heads": G, "dim": d, "vdim": d, "scale": d ** -0.5, "mask": {"size": size["window"], "keep_first": KEEP_FIRST}, "rot": {"base": 10000.0, "dims": d // 4}}
        else:
            H, d, dv = size["gla"]
            for nm, n in (("q", H * d), ("k", H * d), ("v", H * dv)):
                lin(p + nm, n, w)
            mixer = {"heads": H, "dim": d, "vdim": dv, "decay": [1.0 - 2.0 ** (-5.0 - 6.0 * h / H) for h in range(H)], "rot": {"base": 10000.0, "dims": d}}
        lin(p + "g", H * dv, w); lin(p + "o", w, H * dv)
        if mlp == "dense":
            vec(f"l{i}.norm2", w, 1.0)
            lin(f"l{i}.mlp.gate", ff, w); lin(f"l{i}.mlp.up", ff, w); lin(f"l{i}.mlp.down", w, ff)
        layers.append({"type": mix, "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if mlp == "dense" else None})
    return {"architecture": "Luzinex", "vocab": vocab, "width": w, "norm": {"eps": 1e-5}, "layers": layers}, TensorDict(t)


def _make(size_name):
    def make(size, kind, reps, dev):
        from .luzinex import LuzinexModel
        cfg, td = synth(SIZES[size_name], LATENT[size_name], [kind] * reps, device=dev)
        return LuzinexModel(cfg, td, device=dev, dtype=torch.bfloat16)
    return make


def _make_zagilorn(size_name, window):
    def make(size, kind, reps, dev):
        from .zagilorn import ZagilornModel
        cfg, td = latent_bench.synth(dict(SIZES[size_name], window=window), LATENT[size_name], [kind] * reps, device=dev)
        cfg.pop("token_side")                        # the per-layer token input is no part of the comparison
        return ZagilornModel(cfg, td, device=dev, dtype=torch.bfloat16)
    return make


def dual_kernel_legs(size_name: str, prompt: int, ctx: int, dev):
    """Each kernel of the design alone at the size's shapes: time and the fraction of the roofline that bounds it; `like_*`: the like kernel of a closest model on the
    same data where that is another kernel or another form of it."""
    from . import mix_ops
    from .modules import Retention, rotary_frequencies
    from .state_cache import StepBatch
    s, lt = SIZES[size_name], LATENT[size_name]
    out, bf = {}, torch.bfloat16
    rnd = lambda *sh: torch.randn(*sh, device=dev).to(bf)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)
    hbm = lambda by, t: {"us": t * 1e6, "GBps": by / t / 1e9, "of_hbm": by / t / PEAK_HBM}
    flop = lambda fl, t, peak: {"ms": t * 1e3, "tflops": fl / t / 1e12, "of_peak": fl / t / peak}
    n, w = prompt, s["width"]
    cu, seq, pos = i32([0, n]), torch.zeros(n, dtype=torch.int32, device=dev), torch.arange(n, dtype=torch.int32, device=dev)
    sl, la, p0 = i32([0]), i32([n]), i32([0])
    batch = lambda bs: (torch.arange(bs, dtype=torch.int32, device=dev), i32([ctx - 1] * bs), i32([ctx] * bs))

    # latent attention over pages
    H, d, r, dv, rank = lt["heads"], lt["dim"], lt["rot_dim"], lt["vdim"], lt["rank"]
    row, dk, page = rank + r, d + r, 64
    per_seq = -(-max(ctx, n) // page)
    pages = torch.zeros((16 * per_seq, page, row), dtype=bf, device=dev)
    table = torch.randperm(16 * per_seq, device=dev).int().view(16, per_seq).contiguous()
    freq = rotary_frequencies(r, 10000.0)[0].to(dev)
    ckr, z, nw, cq, qw = torch.empty((n, row), dtype=bf, device=dev), rnd(n, Q_RANK + row), torch.ones(rank, device=dev), torch.empty((n, Q_RANK), dtype=bf, device=dev), torch.ones(Q_RANK, device=dev)
    rows = lambda m, sq, ps, slot: mix_ops.latent_rows(sq, ps, slot, 1e-5, freq, 1.0, False, dkv=(ckr[:m], pages, table, z[:m, Q_RANK:], nw), dq=(cq[:m], z[:m, :Q_RANK], qw))
    out["latent_rows_prefill"] = hbm(n * (row * 2 * 3 + Q_RANK * 2 * 2), _time(lambda: rows(n, seq, pos, sl), 20))
    q, k, v, g = rnd(n, H * dk), rnd(n, H * dk), rnd(n, H * dv), rnd(n, H * dv)
    out["rotate_heads_prefill"] = hbm(n * H * r * 2 * 2, _time(lambda: mix_ops.rotate_heads(q, pos, freq, 1.0, False, H, dk, d), 20))
    o = torch.empty((n, H * dv), dtype=bf, device=dev)
    sink = torch.zeros(H, device=dev)
    fl = 2.0 * (dk + dv) * H * n * (n + 1) / 2
    t = _time(lambda: mix_ops.attn_prefill_maps(o, q, k, v, g, None, cu, seq, pos, H, H, 1, dk, dv, dk ** -0.5, 0.0, 1 << 30, mix_ops.MASK_WINDOW, max_rows=n), 10)
    out["attn_prefill_latent_causal_gated"] = flop(fl, t, PEAK_BF16)
    for bs in (1, 16):
        sq, pd, lad = batch(bs)
        out[f"latent_rows_bs{bs}"] = {"us": _time(lambda: rows(bs, sq, pd, sq), 50) * 1e6}
        qd, ql, ol = rnd(bs, H * dk), rnd(H, bs, rank), torch.empty((H, bs, rank), dtype=bf, device=dev)
        out[f"rotate_heads_bs{bs}"] = {"us": _time(lambda: mix_ops.rotate_heads(qd, pd, freq, 1.0, False, H, dk, d), 50) * 1e6}
        by = bs * ctx * row * 2
        out[f"latent_decode_paged_bs{bs}"] = hbm(by, _time(lambda: mix_ops.latent_decode(ol, ql, qd, pages, None, sq, lad, d, r, dk ** -0.5, table=table), 50))
        ring = torch.zeros((16, max(ctx, page), row), dtype=bf, device=dev)
        out[f"like_latent_decode_ring_bs{bs}"] = hbm(by, _time(lambda: mix_ops.latent_decode(ol, ql, qd, ring, sink, sq, lad, d, r, dk ** -0.5), 50))

    # kept-window attention
    H, G, d, W = s["heads"], s["kv_heads"], s["dim"], s["window"]
    wide = rnd(n, (2 * H + G) * d)
    q, k, g = wide[:, : H * d], wide[:, H * d: (H + G) * d], wide[:, (H + G) * d:]
    kr, o, sink = torch.empty((n, G * d), dtype=bf, device=dev), torch.empty((n, H * d), dtype=bf, device=dev), torch.zeros(H, device=dev)
    rk, rv = (torch.zeros((16, KEEP_FIRST + W, G, d), dtype=bf, device=dev) for _ in range(2))
    fq = rotary_frequencies(d // 4, 10000.0)[0].to(dev)
    prep = lambda m, sq, ps, slot, ln: mix_ops.qk_prep(wide[:m, : H * d], wide[:m, H * d: (H + G) * d], wide[:m, H * d: (H + G) * d], None, None, fq, 1.0, True, 0.0, rk, rv, sq, ps, slot,
                                                       ln, d, k_out=kr[:m], keep_first=KEEP_FIRST)
    out["qk_prep_tied_prefill"] = hbm(n * (2 * H + 2 * G) * d * 2 + min(n, W) * 2 * G * d * 2, _time(lambda: prep(n, seq, pos, sl, la), 20))
    pairs = sum(min(i + 1, W) + (KEEP_FIRST if i >= W + KEEP_FIRST else 0) for i in range(n))
    t = _time(lambda: mix_ops.attn_prefill_maps(o, q, kr, k, g, sink, cu, seq, pos, H, G, 1, d, d, d ** -0.5, 0.0, W, mix_ops.MASK_WINDOW, max_rows=n, keep=KEEP_FIRST), 10)
    out["attn_prefill_kept_window_gated"] = flop(4.0 * d * pairs * H, t, PEAK_BF16)
    for bs in (1, 16):
        sq, pd, lad = batch(bs)
        out[f"qk_prep_tied_bs{bs}"] = {"us": _time(lambda: prep(bs, sq, pd, sq, lad), 50) * 1e6}
        od = torch.empty((bs, H * d), dtype=bf, device=dev)
        by = bs * min(ctx, W + KEEP_FIRST) * G * d * 2 * 2
        out[f"attn_decode_kept_window_bs{bs}"] = hbm(by, _time(lambda: mix_ops.attn_decode_maps(od, q[:bs], rk, rv, g[:bs], sink, sq, lad, H, 1, d ** -0.5, 0.0, mix_ops.MASK_WINDOW), 50))

    # retention
    H, d, dv = s["gla"]
    wide = rnd(n, 2 * H * d + 2 * H * dv)
    q, k, v, g = wide[:, : H * d], wide[:, H * d: 2 * H * d], wide[:, 2 * H * d: 2 * H * d + H * dv], wide[:, 2 * H * d + H * dv:]
    decay = [1.0 - 2.0 ** (-5.0 - 6.0 * h / H) for h in range(H)]
    pw = (torch.tensor(decay, dtype=torch.float64)[:, None] ** torch.arange(mix_ops.RETENTION_TILE + 1, dtype=torch.float64)[None]).float().to(dev).contiguous()
    fr = rotary_frequencies(d, 10000.0)[0].to(dev)
    state, o = torch.zeros((16, H, d, dv), device=dev), torch.empty((n, H, dv), device=dev)
    segs = Retention(w, H, d, dv, decay, d, 10000.0, 1e-5).segments(StepBatch(n, 1, False, n, None, cu, seq, pos, sl, p0, la))
    fl = 4.0 * d * dv * H * n
    for name, sg in (("retention_prefill_segmented", segs), ("retention_prefill_one_chain", None)):
        t = _time(lambda: mix_ops.retention(o, state, q, k, v, pw, fr, False, cu, sl, p0, d ** -0.5, segments=sg), 5)
        out[name] = dict(flop(fl, t, PEAK_F32), segments=sg)
    a = torch.empty((n, H * dv), dtype=bf, device=dev)
    out["head_norm_gate_prefill"] = hbm(n * H * dv * (4 + 2 + 2), _time(lambda: mix_ops.head_norm_gate(a, o, None, g, mix_ops.GATE_SILU, 1e-5), 20))
    for bs in (1, 16):
        sq, pd, lad = batch(bs)
        t = _time(lambda: mix_ops.retention_step(a[:bs], state, q[:bs], k[:bs], v[:bs], g[:bs], pw, fr, False, pd, sq, H, d ** -0.5, 1e-5), 50)
        out[f"retention_step_bs{bs}"] = hbm(bs * H * d * dv * 4 * 2, t)

    # what every layer has
    x, y = torch.randn(n, w, device=dev), rnd(n, w)
    h1, h2, w1 = torch.empty((n, w), dtype=bf, device=dev), torch.empty((n, w), dtype=bf, device=dev), torch.ones(w, device=dev)
    out["residual_norm_pair"] = hbm(n * w * (4 + 4 + 2 + 2 + 2), _time(lambda: mix_ops.residual_norm_pair(x, y, mix_ops.RES_ADD, w1, h1, w1, h2, 1e-5), 20))
    ff = gated_ff(s)
    z, a = rnd(n, 2 * ff), torch.empty((n, w + ff), dtype=bf, device=dev)[:, w:]
    out["gelu_glu"] = hbm(n * ff * 6, _time(lambda: mix_ops.glu_act(a, z[:, :ff], z[:, ff:], mix_ops.GLU_GELU_TANH), 20))
    return out


def run(args) -> int:
    dev = torch.device("cuda:0")
    torch.cuda.set_device(dev)
    from . import _lib
    _lib.mixlib()
    prompt, ctx = args.prefill_tokens, 1000
    res = {"metric": "dual_family_layer_times", "unit": "ms per layer", "dtype": "bf16", "data": "synthetic", "prompt": prompt, "ctx": ctx, "sizes": {}}
    for name in (args.mixer_sizes.split(",") if args.mixer_sizes else list(SIZES)):
        t0 = time.time()
        entry = {"gated_ff": gated_ff(SIZES[name]), "latent": LATENT[name], "q_rank": Q_RANK,
                 "luzinex_layers": model_legs(name, prompt, ctx, args.steps, dev, kinds=KINDS, make=_make(name)), "kernels": dual_kernel_legs(name, prompt, ctx, dev)}
        try:
            entry["closest_model_zagilorn_layers"] = model_legs(name, prompt, ctx, args.steps, dev, kinds=[("latent_attention", "dense")], make=_make_zagilorn(name, max(prompt, ctx)))
            entry["closest_model_vofanex_layers"] = model_legs(name, prompt, ctx, args.steps, dev, kinds=[("attention", "dense"), ("gla", "dense")])
            entry["closest_model_vofanex_kernels"] = kernel_legs(name, prompt, ctx, dev)
            entry["closest_model_zagilorn_kernels"] = latent_bench.latent_kernel_legs(name, prompt, ctx, dev)
        except Exception as e:                       # the comparison leg must not hide the new design's numbers
            entry["closest_model_error"] = f"{type(e).__name__}: {e}"
        entry["seconds"] = round(time.time() - t0, 1)
        res["sizes"][name] = entry
    print(json.dumps(res))
    return 0
