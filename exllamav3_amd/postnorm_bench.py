"""
`bench.py --postnorm-family`: prefill and decode throughput of Menerax layers (post-norm blocks: paged latent attention with a gate per head, or kept-window attention with
short convolutions and soft-capped scores beside time mixing, over a clamped-swish feed-forward; random weights) at sizes that resemble real models' layers, beside the
closest existing models of the same library, timed in the same process at the same width, head shapes and weight counts -- Luzinex's latent layer, and its
window and retention layers one behind the other -- and each kernel of the design alone against its roofline, next to the like kernel of those models and of Vofanex
(gated linear attention).  Prints one JSON line; the default workload of bench.py and the JSON line it prints are untouched.
"""
from __future__ import annotations
import json
import math
import time
import torch
from . import dual_bench
from .dual_bench import KEEP_FIRST, Q_RANK, gated_ff
from .latent_bench import LATENT
from .mixer_bench import PEAK_BF16, PEAK_F32, PEAK_HBM, SIZES, TensorDict, _time, kernel_legs, model_legs

KINDS = [("latent_attention", "dense"), ("parallel", "dense")]
TAPS, RANK, SOFTCAP, LIMIT = 4, 64, 30.0, 7.0


def mix_heads(size: dict) -> tuple[int, int]:
    """Time-mixing heads of 64 channels over the model's width."""
    d = size.get("mix_dim", 64)
    return size["width"] // d, d


def synth(size: dict, lt: dict, kinds, vocab=32000, seed=0, device="cuda:0", share=False):
    """Random Menerax weights and their config: size as in mixer_bench.SIZES, lt as in latent_bench.LATENT (q_rank: Q_RANK if it has none).  share: the list of layers
    runs twice, the second time with the first one's weights."""
    g = torch.Generator(device=device).manual_seed(seed)
    w, t, layers, ff = size["width"], {}, [], gated_ff(size)
    q_rank = lt.get("q_rank", Q_RANK)

    def lin(name, o, i, s=1.0):
        t[name] = (torch.randn(o, i, generator=g, device=device) * (s / math.sqrt(i))).to(torch.bfloat16)

    def vec(name, n, mean=0.0, s=0.1):
        t[name] = (mean + s * torch.randn(n, generator=g, device=device)).to(torch.bfloat16)
    lin("embed", vocab, w, math.sqrt(w)); lin("head", vocab, w); vec("embed.norm", w); vec("final.norm", w)
    for i, (mix, mlp) in enumerate(kinds):
        p = f"l{i}.mix."
        vec(f"l{i}.norm1", w)
        if mix == "latent_attention":
            H, d, r, dv, rank = lt["heads"], lt["dim"], lt["rot_dim"], lt["vdim"], lt["rank"]
            lin(p + "dq", q_rank, w); vec(p + "dq.norm", q_rank, 1.0); lin(p + "uq", H * (d + r), q_rank)
            lin(p + "uk", H * d, rank); lin(p + "uv", H * dv, rank)
            lin(p + "dkv", rank + r, w); vec(p + "dkv.norm", rank, 1.0)
            lin(p + "g", H, w); lin(p + "o", w, H * dv)
            mixer = {"heads": H, "dim": d, "rot_dim": r, "vdim": dv, "kv_rank": rank, "q_rank": q_rank, "scale": (d + r) ** -0.5, "rot": {"base": 10000.0, "dims": r}}
        else:
            H, G, d = size["heads"], size["kv_heads"], size["dim"]
            a = p + "left."
            for nm, n in (("q", H * d), ("k", G * d), ("v", G * d)):
                lin(a + nm, n, w); vec(a + nm + ".b", n); vec(a + nm + ".conv", n * TAPS, 0.25); t[a + nm + ".conv"] = t[a + nm + ".conv"].view(n, TAPS)
            vec(a + "q.norm", d, 1.0); vec(a + "k.norm", d, 1.0); lin(a + "g", H * d, w); lin(a + "o", w, H * d)
            b, (Hm, dm) = p + "right.", mix_heads(size)
            n = Hm * dm
            for nm in "rkvg":
                lin(b + nm, n, w)
            for nm in "rkvgw":
                vec(b + "mu." + nm, w, 0.5)
            lin(b + "w1", RANK, w); lin(b + "w2", n, RANK); vec(b + "w0", n, -3.0, 1.0); vec(b + "u", n, 0.5); t[b + "u"] = t[b + "u"].view(Hm, dm); vec(b + "norm", n, 1.0); lin(b + "o", w, n)
            mixer = {"left": {"heads": H, "kv_heads": G, "dim": d, "vdim": d, "conv": TAPS, "scale": d ** -0.5, "softcap": SOFTCAP, "mask": {"size": size["window"], "keep_first": KEEP_FIRST},
                              "rot": {"base": 500000.0, "dims": d // 2, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}},
                     "right": {"heads": Hm, "dim": dm}, "left_scale": 0.9, "right_scale": 1.3}
        if mlp == "dense":
            vec(f"l{i}.norm2", w)
            lin(f"l{i}.mlp.gate", ff, w); lin(f"l{i}.mlp.up", ff, w); lin(f"l{i}.mlp.down", w, ff)
        layers.append({"type": mix, "mixer": mixer, "mlp": {"kind": "dense", "ff": ff, "limit": LIMIT} if mlp == "dense" else None})
    if share:
        layers += [dict(L, weights_of=i) for i, L in enumerate(layers)]
    return {"architecture": "Menerax", "vocab": vocab, "width": w, "norm": {"eps": 1e-5}, "layers": layers}, TensorDict(t)


def _make(size_name):
    def make(size, kind, reps, dev):
        from .menerax import MeneraxModel
        cfg, td = synth(SIZES[size_name], LATENT[size_name], [kind] * reps, device=dev)
        return MeneraxModel(cfg, td, device=dev, dtype=torch.bfloat16)
    return make


def postnorm_kernel_legs(size_name: str, prompt: int, ctx: int, dev):
    """Each kernel of the design alone at the size's shapes: time and the fraction of the roofline that bounds it; `like_*`: the like kernel of a closest model on the
    same data where that is another kernel or another form of it."""
    from . import mix_ops
    from .modules import TimeMix, rotary_frequencies
    from .state_cache import StepBatch
    s, lt = SIZES[size_name], LATENT[size_name]
    out, bf = {}, torch.bfloat16
    rnd = lambda *sh: torch.randn(*sh, device=dev).to(bf)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)
    hbm = lambda by, t: {"us": t * 1e6, "GBps": by / t / 1e9, "of_hbm": by / t / PEAK_HBM}
    flop = lambda fl, t, peak: {"ms": t * 1e3, "tflops": fl / t / 1e12, "of_peak": fl / t / peak}
    n, w = prompt, s["width"]

    def batch(lens, pos0):
        b = len(lens)
        cu = [0]
        for l in lens:
            cu.append(cu[-1] + l)
        seq = torch.repeat_interleave(torch.arange(b), torch.tensor(lens)).int().to(dev)
        pos = torch.cat([torch.arange(p, p + l) for p, l in zip(pos0, lens)]).int().to(dev)
        return StepBatch(cu[-1], b, pos0[0] > 0, max(lens), None, i32(cu), seq, pos, torch.arange(b, dtype=torch.int32, device=dev), i32(pos0), i32([p + l for p, l in zip(pos0, lens)]))
    whole = batch([n], [0])
    decode = {bs: batch([1] * bs, [ctx - 1] * bs) for bs in (1, 16)}

    # convolved, normed, rotated queries and keys; soft-capped attention over the kept window
    H, G, d, W = s["heads"], s["kv_heads"], s["dim"], s["window"]
    C = (H + 2 * G) * d
    wide, z = rnd(n, C + H * d), torch.empty((n, C), dtype=bf, device=dev)
    x, g = wide[:, :C], wide[:, C:]
    cw, nw = torch.randn(TAPS, C, device=dev), torch.ones(d, device=dev)
    ring = torch.zeros((16, TAPS - 1, C), dtype=bf, device=dev)
    rk, rv = (torch.zeros((16, KEEP_FIRST + W, G, d), dtype=bf, device=dev) for _ in range(2))
    fq = rotary_frequencies(d // 2, 500000.0)[0].to(dev)
    prep = lambda sb: mix_ops.conv_prep(z[: sb.n], x[: sb.n], cw, ring, nw, nw, fq, 1.0, False, 1e-5, rk, rv, sb, H, keep_first=KEEP_FIRST)
    out["conv_prep_prefill"] = hbm(n * C * 2 * 2 + min(n, W) * 2 * G * d * 2, _time(lambda: prep(whole), 20))
    like = lambda sb: mix_ops.qk_prep(x[: sb.n, : H * d], x[: sb.n, H * d: (H + G) * d], x[: sb.n, (H + G) * d:], nw, nw, fq, 1.0, False, 1e-5, rk, rv, sb.tok_seq, sb.tok_pos, sb.slots,
                                      sb.len_after, d, keep_first=KEEP_FIRST)
    out["like_qk_prep_prefill"] = hbm(n * (H + G) * d * 2 * 2 + min(n, W) * 2 * G * d * 2 * 2, _time(lambda: like(whole), 20))
    q, k, v = z[:, : H * d], z[:, H * d: (H + G) * d], z[:, (H + G) * d:]
    prep(whole)
    o = torch.empty((n, H * d), dtype=bf, device=dev)
    pairs = sum(min(i + 1, W) + (KEEP_FIRST if i >= W + KEEP_FIRST else 0) for i in range(n))
    attn = lambda cap: _time(lambda: mix_ops.attn_prefill_maps(o, q, k, v, g, None, whole.cu, whole.tok_seq, whole.tok_pos, H, G, 1, d, d, d ** -0.5, cap, W, mix_ops.MASK_WINDOW, max_rows=n,
                                                               keep=KEEP_FIRST, out_scale=0.9), 10)
    out["attn_prefill_kept_window_softcap"] = flop(4.0 * d * pairs * H, attn(SOFTCAP), PEAK_BF16)
    out["like_attn_prefill_kept_window"] = flop(4.0 * d * pairs * H, attn(0.0), PEAK_BF16)
    for bs, sb in decode.items():
        out[f"conv_prep_bs{bs}"] = {"us": _time(lambda: prep(sb), 50) * 1e6}
        out[f"like_qk_prep_bs{bs}"] = {"us": _time(lambda: like(sb), 50) * 1e6}
        by = bs * min(ctx, W + KEEP_FIRST) * G * d * 2 * 2
        for nm, cap in (("attn_decode_kept_window_softcap", SOFTCAP), ("like_attn_decode_kept_window", 0.0)):
            out[f"{nm}_bs{bs}"] = hbm(by, _time(lambda: mix_ops.attn_decode_maps(o[:bs], q[:bs], rk, rv, g[:bs], None, sb.slots, sb.len_after, H, 1, d ** -0.5, cap, mix_ops.MASK_WINDOW), 50))

    # time mixing
    Hm, dm = mix_heads(s)
    N = Hm * dm
    h, mix, last, mu = rnd(n, w), torch.empty((5, n, w), dtype=bf, device=dev), torch.zeros((16, w), dtype=bf, device=dev), torch.rand(5, w, device=dev)
    out["token_shift_prefill"] = hbm(n * w * 2 * 6, _time(lambda: mix_ops.token_shift(mix, h, last, mu, whole), 20))
    t, w2, w0 = rnd(n, RANK), (rnd(N, RANK).float() / 8).to(bf), torch.randn(N, device=dev) - 3.0
    log2w = torch.empty((n, N), dtype=torch.float32, device=dev)
    out["decay_log2_prefill"] = hbm(n * (N * 4 + RANK * 2), _time(lambda: mix_ops.decay_log2(log2w, t, w2, w0), 20))
    out["decay_log2_prefill"]["float32_tflops"] = 2.0 * n * N * RANK / out["decay_log2_prefill"]["us"] / 1e6
    rkvg = rnd(4, n, N)
    u, nrm = torch.rand(N, device=dev), torch.ones(N, device=dev)
    state, a = torch.zeros((16, Hm, dm, dm), device=dev), torch.empty((n, N), dtype=bf, device=dev)
    segs = TimeMix(w, Hm, dm, 1e-5).segments(whole)
    fl = 4.0 * dm * dm * Hm * n
    for name, sg in (("timemix_prefill_segmented", segs), ("timemix_prefill_one_chain", None)):
        tt = _time(lambda: mix_ops.timemix(None, a, rkvg[3], nrm, 1e-5, state, rkvg[0], rkvg[1], rkvg[2], log2w, u, whole.cu, whole.slots, whole.pos0, segments=sg), 5)
        out[name] = dict(flop(fl, tt, PEAK_F32), segments=sg, of_hbm_one_pass=n * N * (2 * 4 + 4 + 2) / tt / PEAK_HBM)
    for bs, sb in decode.items():
        few = torch.empty((5, bs, w), dtype=bf, device=dev)
        out[f"token_shift_bs{bs}"] = {"us": _time(lambda: mix_ops.token_shift(few, h[:bs], last, mu, sb), 50) * 1e6}
        tt = _time(lambda: mix_ops.timemix_step(a[:bs], state, rkvg[0, :bs], rkvg[1, :bs], rkvg[2, :bs], rkvg[3, :bs], t[:bs], w2, w0, u, nrm, sb.tok_pos, sb.slots, 1e-5), 50)
        out[f"timemix_step_bs{bs}"] = hbm(bs * Hm * dm * dm * 4 * 2, tt)
    # products of few rows: weights of several layers in turn (none of them still cached), beside the vendor's
    for bs in (1, 16):
        for nm, rows, K in (("qkvg", C + H * d, w), ("ff_down", w, gated_ff(s))):
            ws = [rnd(rows, K) for _ in range(max(2, int(6e8 / (rows * K * 2))))]
            xs = rnd(bs, K)
            for label, f in (("skinny", lambda x_, w_: mix_ops.skinny(x_, w_)), ("like_vendor", torch.nn.functional.linear)):
                out[f"{label}_{nm}_bs{bs}"] = hbm(rows * K * 2, _time(lambda: [f(xs, x_) for x_ in ws], 10) / len(ws))
            del ws
        ws, xs = [rnd(4 * N + RANK, w) for _ in range(3)], rnd(5, bs, w)
        out[f"skinny_stack_rkvg_w1_bs{bs}"] = hbm(ws[0].numel() * 2, _time(lambda: [mix_ops.skinny_stack(xs, x_, N) for x_ in ws], 10) / 3)
        del ws

    # latent attention's gate per head, and what every layer has
    Hl, dl, r, dv = lt["heads"], lt["dim"], lt["rot_dim"], lt["vdim"]
    dk = dl + r
    ql, kl, vl, gl, ol = rnd(n, Hl * dk), rnd(n, Hl * dk), rnd(n, Hl * dv), rnd(n, Hl), torch.empty((n, Hl * dv), dtype=bf, device=dev)
    tt = _time(lambda: mix_ops.attn_prefill_maps(ol, ql, kl, vl, gl, None, whole.cu, whole.tok_seq, whole.tok_pos, Hl, Hl, 1, dk, dv, dk ** -0.5, 0.0, 1 << 30, mix_ops.MASK_WINDOW, max_rows=n), 10)
    out["attn_prefill_latent_causal_head_gate"] = flop(2.0 * (dk + dv) * Hl * n * (n + 1) / 2, tt, PEAK_BF16)
    for bs in (1, 16):
        oh = rnd(Hl, bs, dv)
        out[f"heads_gate_by_head_bs{bs}"] = {"us": _time(lambda: mix_ops.heads_gate(ol[:bs], oh, dv, bs * dv, gl[:bs], Hl, dv), 50) * 1e6}
    xr, y, hc, wn = torch.randn(n, w, device=dev), rnd(n, w), torch.empty((n, w), dtype=bf, device=dev), torch.ones(w, device=dev)
    out["residual_post_norm"] = hbm(n * w * (4 + 4 + 2 + 2), _time(lambda: mix_ops.residual_norm(xr, y, mix_ops.RES_ADD, wn, 1e-5, mix_ops.OUT_CAST, 0.0, None, None, hc), 20))
    h2 = torch.empty_like(hc)
    out["like_residual_norm_pair"] = hbm(n * w * (4 + 4 + 2 + 2 + 2), _time(lambda: mix_ops.residual_norm_pair(xr, y, mix_ops.RES_ADD, wn, hc, wn, h2, 1e-5), 20))
    for bs in (1, 16):
        out[f"residual_post_norm_bs{bs}"] = {"us": _time(lambda: mix_ops.residual_norm(xr[:bs], y[:bs], mix_ops.RES_ADD, wn, 1e-5, mix_ops.OUT_CAST, 0.0, None, None, hc[:bs]), 50) * 1e6}
    table, toks = rnd(32000, w), torch.randint(0, 32000, (n,), device=dev).int()
    out["embed_norm"] = hbm(n * w * (2 + 4 + 2), _time(lambda: mix_ops.embed_norm(xr, hc, table, toks, wn, 1e-5), 20))
    ff = gated_ff(s)
    zz, af = rnd(n, 2 * ff), torch.empty((n, ff), dtype=bf, device=dev)
    out["clamped_swish_glu"] = hbm(n * ff * 6, _time(lambda: mix_ops.glu_act(af, zz[:, :ff], zz[:, ff:], mix_ops.GLU_CLAMPED_SWISH, LIMIT), 20))
    return out


def run(args) -> int:
    dev = torch.device("cuda:0")
    torch.cuda.set_device(dev)
    from . import _lib
    _lib.mixlib()
    prompt, ctx = args.prefill_tokens, 1000
    res = {"metric": "postnorm_family_layer_times", "unit": "ms per layer", "dtype": "bf16", "data": "synthetic", "prompt": prompt, "ctx": ctx, "sizes": {}}
    for name in (args.mixer_sizes.split(",") if args.mixer_sizes else list(SIZES)):
        t0 = time.time()
        entry = {"gated_ff": gated_ff(SIZES[name]), "latent": LATENT[name], "q_rank": Q_RANK, "time_mix_heads": mix_heads(SIZES[name]),
                 "menerax_layers": model_legs(name, prompt, ctx, args.steps, dev, kinds=KINDS, make=_make(name)), "kernels": postnorm_kernel_legs(name, prompt, ctx, dev)}
        try:
            entry["closest_model_luzinex_layers"] = model_legs(name, prompt, ctx, args.steps, dev, kinds=[("latent_attention", "dense"), ("attention", "none"), ("retention", "dense")],
                                                               make=dual_bench._make(name))
            entry["closest_model_luzinex_kernels"] = dual_bench.dual_kernel_legs(name, prompt, ctx, dev)
            entry["closest_model_vofanex_kernels"] = kernel_legs(name, prompt, ctx, dev)
        except Exception as e:                       # the comparison leg must not hide the new design's numbers
            entry["closest_model_error"] = f"{type(e).__name__}: {e}"
        entry["seconds"] = round(time.time() - t0, 1)
        res["sizes"][name] = entry
    print(json.dumps(res))
    return 0
