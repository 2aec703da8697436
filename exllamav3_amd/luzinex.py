"""
Luzinex: a decoder-only model of parallel blocks with two norms over a float32 stream, x <- x + mixer(norm1(x)) + ff(norm2(x)).  A layer's mixer is latent
attention over every earlier token (a cached low-rank latent and one rotated key part per token, queries through a latent of their own, element-wise output
gate; a layer may read an earlier layer's cached rows), sliding-window attention that keeps the first tokens of a sequence visible (values are the keys before
rotation, a sink, element-wise output gate), or retention (linear attention with a fixed decay per head).  The feed-forward is a gated gelu layer or none.  The
order of layers and every size and constant come from config.json:

    architecture "Luzinex"; vocab; width; norm.eps
    layers[i]: type "latent_attention": mixer {heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, rot {base, dims}, kv_from (optional)}
               type "attention":        mixer {heads, kv_heads, dim, vdim, scale, mask {size, keep_first}, rot {base, dims}}
               type "retention":        mixer {heads, dim, vdim, decay [heads], rot {base, dims}}
               mlp: null | {"kind": "dense", ff}

Tensor names: embed, head, final.norm, l<i>.norm1, l<i>.norm2; latent l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,g,o} (no dkv with kv_from); attention
l<i>.mix.{q,k,sink,g,o}; retention l<i>.mix.{q,k,v,g,o}; l<i>.mlp.{gate,up,down}.

The model is a list of DualNormBlock over the mechanisms of modules.py; its state is a SlotStateCache with one entry per layer (a layer that reads another's rows
has none and is given that layer's); `step` is the one function the generator, the command line and the trace runner call.
"""
from __future__ import annotations
import json
import os
import torch
import torch.nn.functional as F
from . import mix_ops
from .loader import SafetensorsCollection
from .modules import DualNormBlock, GatedMLP, KeptWindowAttention, PagedLatentAttention, Retention, _f32, _w
from .state_cache import SlotStateCache, StepBatch


class LuzinexConfig:
    def __init__(self, d: dict):
        self.vocab = int(d["vocab"])
        self.width = int(d["width"])
        self.eps = float(d["norm"]["eps"])
        self.layers = d["layers"]
        if not self.layers:
            raise RuntimeError("Luzinex: config has no layers")
        self.source = []                         # layer -> the layer whose cached state it uses
        for i, L in enumerate(self.layers):
            j = L["mixer"].get("kv_from")
            j = i if j is None else int(j)
            if j != i:
                if not 0 <= j < i or self.layers[j]["type"] != "latent_attention" or L["type"] != "latent_attention" or self.layers[j]["mixer"].get("kv_from") is not None:
                    raise RuntimeError(f"Luzinex: layer {i} reads the latent of layer {j}, which has none of its own")
                a, b = L["mixer"], self.layers[j]["mixer"]
                if any(a[key] != b[key] for key in ("kv_rank", "rot_dim", "rot")):
                    raise RuntimeError(f"Luzinex: layer {i} reads the latent of layer {j}, whose rank or rotation is another")
            self.source.append(j)

    def _mixer(self, i: int, L: dict):
        m, w = L["mixer"], self.width
        rot = m["rot"]
        base = float(rot["base"])
        if L["type"] == "latent_attention":
            return PagedLatentAttention(w, int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"]), int(m["q_rank"]), float(m["scale"]), self.eps,
                                        int(rot.get("dims", m["rot_dim"])), base, interleaved=False, sink=False, gate=True, layer=i,
                                        kv_from=None if self.source[i] == i else self.source[i])
        if L["type"] == "attention":
            mask = m["mask"]
            return KeptWindowAttention(w, int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]), int(m.get("vdim", m["dim"])), float(m["scale"]), int(mask["size"]),
                                       int(mask.get("keep_first", 0)), int(rot.get("dims", m["dim"])), base, interleaved=True, tied=True, sink=True, gate=True)
        if L["type"] == "retention":
            return Retention(w, int(m["heads"]), int(m["dim"]), int(m.get("vdim", m["dim"])), m["decay"], int(rot.get("dims", m["dim"])), base, self.eps, interleaved=False)
        raise RuntimeError(f"Luzinex: layer {i} has an unknown mixer type {L['type']!r}")

    def _mlp(self, i: int, L: dict):
        f = L.get("mlp")
        if f is None:
            return None
        if f["kind"] == "dense":
            return GatedMLP(self.width, int(f["ff"]), "gelu_tanh")
        raise RuntimeError(f"Luzinex: layer {i} has an unknown feed-forward kind {f['kind']!r}")

    def build_blocks(self) -> list[DualNormBlock]:
        return [DualNormBlock(self.width, self.eps, self._mixer(i, L), self._mlp(i, L)) for i, L in enumerate(self.layers)]


class LuzinexModel:
    architecture = "Luzinex"
    native_libraries = ("mix",)          # what a fresh checkout has to compile before this model runs
    PAGE_SIZE = 64

    def __init__(self, config: dict, stc, device="cuda:0", dtype=torch.bfloat16):
        if dtype not in (torch.bfloat16, torch.float32):
            raise RuntimeError("Luzinex runs in bfloat16 or float32")
        self.cfg = LuzinexConfig(config)
        self.device, self.dtype = torch.device(device), dtype
        self.vocab = self.cfg.vocab
        self.blocks = self.cfg.build_blocks()
        for i, blk in enumerate(self.blocks):
            blk.load(stc, f"l{i}.", dtype, self.device)
        self.embed = _w(stc, "embed", dtype, self.device)
        self.head = _w(stc, "head", dtype, self.device)
        self.final_w = _f32(stc, "final.norm", self.device)
        w = self.cfg.width
        assert self.embed.shape == (self.vocab, w) and self.head.shape == (self.vocab, w) and self.final_w.numel() == w
        self.layer_taps = None               # diagnostics: a list that receives a copy of the residual after every layer

    @classmethod
    def from_directory(cls, directory: str, device="cuda:0", dtype=torch.bfloat16) -> "LuzinexModel":
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
        mix_ops.embed_copy(x, None, self.embed, sb.tokens)
        y = None
        for i, blk in enumerate(self.blocks):
            h1, h2 = blk.inputs(x, y, mix_ops.RES_KEEP if y is None else mix_ops.RES_ADD)
            if self.layer_taps is not None and i:
                self.layer_taps.append(x.clone())
            y = blk.forward(h1, h2, sb, cache.layers[self.cfg.source[i]])
        sb.shared.clear()
        mix_ops.residual_norm_pair(x, y, mix_ops.RES_ADD, None, None, None, None, self.cfg.eps)
        if self.layer_taps is not None:
            self.layer_taps.append(x.clone())
        if sb.want_rows is None or sb.want_rows.numel() == 0:
            return None
        hw = torch.empty((sb.want_rows.numel(), w), dtype=self.dtype, device=self.device)
        mix_ops.rms_norm_rows(hw, x, sb.want_rows, self.final_w, self.cfg.eps)
        return F.linear(hw, self.head).float()
