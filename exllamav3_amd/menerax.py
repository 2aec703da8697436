"""
Menerax: a decoder-only model of post-norm blocks over a float32 stream: x += norm1(mixer(x)); x += norm2(ff(x)), with the norms behind the sublayers and no norm
ahead of them.  A layer's mixer is latent attention over every earlier token (a cached low-rank latent and one rotated key part per token, queries
through a latent of their own, one output gate per head), or two mixers side by side, scaled and added: sliding-window attention that keeps the first tokens of a
sequence visible (biases, short convolutions on q / k / v, normed queries and keys, soft-capped scores, element-wise output gate) and RWKV-style time mixing.  The
feed-forward is a gated layer with a clamped swish, or none.  A layer may use an earlier one's weights with a cache of its own.  The order of layers and every size and
constant come from config.json:

    architecture "Menerax"; vocab; width; norm.eps
    layers[i]: type "latent_attention": mixer {heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, rot {base, dims}}
               type "parallel":         mixer {left {heads, kv_heads, dim, vdim, conv, scale, softcap, mask {size, keep_first}, rot {base, dims, scaling {factor, low, high, original}}},
                                               right {heads, dim}, left_scale, right_scale}
               mlp: null | {"kind": "dense", ff, limit};  weights_of (optional): the layer whose tensors this layer uses

Tensor names: embed, embed.norm, head, final.norm, l<i>.norm1, l<i>.norm2; latent l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,g,o}; parallel
l<i>.mix.left.{q,k,v (with .b and .conv),q.norm,k.norm,g,o} and l<i>.mix.right.{mu.r,mu.k,mu.v,mu.g,mu.w,r,k,v,g,w1,w2,w0,u,norm,o}; l<i>.mlp.{gate,up,down}.  The stored
weights of norm1, norm2, embed.norm and final.norm are deviations from one.

The model is a list of PostNormBlock over the mechanisms of modules.py (a shared layer is the same block twice); its state is a SlotStateCache with one entry per layer;
`step` is the one function the generator, the command line and the trace runner call.
"""
from __future__ import annotations
import json
import os
import torch
import torch.nn.functional as F
from . import mix_ops
from .loader import SafetensorsCollection
from .modules import GatedMLP, KeptWindowAttention, PagedLatentAttention, PostNormBlock, SummedMixers, TimeMix, _f32, _w
from .state_cache import SlotStateCache, StepBatch


class MeneraxConfig:
    def __init__(self, d: dict):
        self.vocab = int(d["vocab"])
        self.width = int(d["width"])
        self.eps = float(d["norm"]["eps"])
        self.layers = d["layers"]
        if not self.layers:
            raise RuntimeError("Menerax: config has no layers")
        self.weights_of = [self._owner(i) for i in range(len(self.layers))]         # layer -> the layer whose tensors it uses

    def _owner(self, i: int) -> int:
        L, seen = self.layers[i], {i}
        while (j := self.layers[i].get("weights_of")) is not None:
            i = int(j)
            if not 0 <= i < len(self.layers) or i in seen:
                raise RuntimeError(f"Menerax: weights_of {j} names no layer with tensors of its own")
            seen.add(i)
            if any(key in L and L[key] != self.layers[i].get(key) for key in ("type", "mixer", "mlp")):
                raise RuntimeError(f"Menerax: a layer uses the weights of layer {i} but describes another layer")
        return i

    def _mixer(self, i: int, L: dict):
        m, w = L["mixer"], self.width
        if L["type"] == "latent_attention":
            rot = m["rot"]
            return PagedLatentAttention(w, int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"]), int(m["q_rank"]), float(m["scale"]), self.eps,
                                        int(rot.get("dims", m["rot_dim"])), float(rot["base"]), rot.get("scaling"), interleaved=True, sink=False, gate=True, layer=i, gate_per_head=True)
        if L["type"] == "parallel":
            a, r = m["left"], m["right"]
            mask, rot = a["mask"], a["rot"]
            left = KeptWindowAttention(w, int(a["heads"]), int(a.get("kv_heads", a["heads"])), int(a["dim"]), int(a.get("vdim", a["dim"])), float(a["scale"]), int(mask["size"]),
                                       int(mask.get("keep_first", 0)), int(rot.get("dims", a["dim"])), float(rot["base"]), interleaved=False, sink=False, gate=True, bias=True,
                                       taps=int(a["conv"]), qk_norm=True, softcap=float(a["softcap"]), rot_scaling=rot.get("scaling"), eps=self.eps, out_scale=float(m["left_scale"]))
            return SummedMixers(w, left, TimeMix(w, int(r["heads"]), int(r["dim"]), self.eps, out_scale=float(m["right_scale"])))
        raise RuntimeError(f"Menerax: layer {i} has an unknown mixer type {L['type']!r}")

    def _mlp(self, i: int, L: dict):
        f = L.get("mlp")
        if f is None:
            return None
        if f["kind"] == "dense":
            return GatedMLP(self.width, int(f["ff"]), "clamped_swish", limit=float(f["limit"]))
        raise RuntimeError(f"Menerax: layer {i} has an unknown feed-forward kind {f['kind']!r}")

    def build_blocks(self) -> dict[int, PostNormBlock]:
        """The blocks that have tensors of their own, by layer."""
        return {i: PostNormBlock(self.width, self.eps, self._mixer(i, self.layers[i]), self._mlp(i, self.layers[i])) for i in sorted(set(self.weights_of))}


class MeneraxModel:
    architecture = "Menerax"
    native_libraries = ("mix",)          # what a fresh checkout has to compile before this model runs
    PAGE_SIZE = 64

    def __init__(self, config: dict, stc, device="cuda:0", dtype=torch.bfloat16):
        if dtype not in (torch.bfloat16, torch.float32):
            raise RuntimeError("Menerax runs in bfloat16 or float32")
        self.cfg = MeneraxConfig(config)
        self.device, self.dtype = torch.device(device), dtype
        self.vocab = self.cfg.vocab
        own = self.cfg.build_blocks()
        for i, blk in own.items():
            blk.load(stc, f"l{i}.", dtype, self.device)
        self.blocks = [own[j] for j in self.cfg.weights_of]
        self.embed = _w(stc, "embed", dtype, self.device)
        self.head = _w(stc, "head", dtype, self.device)
        self.embed_norm, self.final_norm = ((1.0 + _f32(stc, nm, self.device)).contiguous() for nm in ("embed.norm", "final.norm"))
        w = self.cfg.width
        assert self.embed.shape == (self.vocab, w) and self.head.shape == (self.vocab, w) and self.final_norm.numel() == w == self.embed_norm.numel()
        self.layer_taps = None               # diagnostics: a list that receives a copy of the residual after every layer

    @classmethod
    def from_directory(cls, directory: str, device="cuda:0", dtype=torch.bfloat16) -> "MeneraxModel":
        with open(os.path.join(directory, "config.json")) as f:
            config = json.load(f)
        return cls(config, SafetensorsCollection(directory), device=device, dtype=dtype)

    def new_cache(self, slots: int = 4, tokens: int = 0) -> SlotStateCache:
        """tokens: the most tokens alive at once, if known (sizes the pages of the latent layers)."""
        return SlotStateCache([blk.state_specs() for blk in self.blocks], self.device, slots=slots, page_size=self.PAGE_SIZE, tokens=tokens)

    @torch.no_grad()
    def step(self, sb: StepBatch, cache: SlotStateCache) -> torch.Tensor | None:
        """Run the step's rows through every layer over the slots of `cache`; returns float32 logits [wanted rows, vocab] (None if none are wanted)."""
        w, n = self.cfg.width, sb.n
        x = torch.empty((n, w), dtype=torch.float32, device=self.device)
        h = torch.empty((n, w), dtype=self.dtype, device=self.device)
        mix_ops.embed_norm(x, h, self.embed, sb.tokens, self.embed_norm, self.cfg.eps)
        for i, blk in enumerate(self.blocks):
            h = blk.forward(x, h, sb, cache.layers[i], last=i + 1 == len(self.blocks))
            if self.layer_taps is not None:
                self.layer_taps.append(x.clone())
        sb.shared.clear()
        if sb.want_rows is None or sb.want_rows.numel() == 0:
            return None
        hw = torch.empty((sb.want_rows.numel(), w), dtype=self.dtype, device=self.device)
        mix_ops.rms_norm_rows(hw, x, sb.want_rows, self.final_norm, self.cfg.eps)
        return F.linear(hw, self.head).float()
