"""Fidatar: a decoder that norms AFTER the sum — both sublayers of a layer read the fp32 residual stream x itself —

    x <- N(c x + mixer(x)) w1;    x <- N(c x + ff(x)) w2          N(z) = z / sqrt(mean z^2 + eps), c = `postln_alpha`

with two mixers in any order: `mlstm` (a matrix memory with exponential gates) and `attention` (GQA, biases, normed q and k,
half-split partial rotation with YaRN frequencies, queries that see their own block of positions only, a 1 in the softmax
denominator).  The feed-forward is W_down relu(W_up h)^2, dense or a mixture of such units chosen by sigmoid scores among the best
groups of neighbours, or absent.  One more norm, an untied head and soft-capped logits.

config.json gives `width`, `vocab`, `norm.eps`, `embedding.scale`, `postln_alpha`, `logit_softcap` and `layers[i].type|mixer|mlp`;
tensors are named `embed`, `l<i>.norm1|norm2`, `l<i>.mix.*`, `l<i>.mlp.*`, `final.norm`, `head`.  This file only maps those keys and
names onto the mechanisms of utils/mixers.py; the step (ragged: portions of prompts beside decoded tokens), the paged KV pool and the
recurrent state slots are FlashCausalLM's (models/flash_causal_lm.py)."""
import json
from typing import List, Optional

import torch

from tgis_amd import native
from tgis_amd.utils.layers import FastLinear
from tgis_amd.utils.mixers import ActivatedMLP, HalfRotatedBlockAttention, MatrixMemory, PostNormResidual, RoutedExperts

MIXER_TYPES = ("mlstm", "attention")
# what guards the division of a matrix memory's read-out: a constant of the design
MEMORY_READ_EPS = 1e-6


class FidatarConfig:
    model_type = "fidatar"

    def __init__(self, width: int, vocab: int, layers: List[dict], norm: dict, embedding: Optional[dict] = None, postln_alpha: float = 1.0,
                 logit_softcap: Optional[float] = None, **kwargs):
        self.width, self.vocab, self.layers = int(width), int(vocab), layers
        self.eps = float(norm["eps"])
        self.embedding_scale = float((embedding or {}).get("scale", 1.0))
        self.postln_alpha = float(postln_alpha)
        self.logit_softcap = float(logit_softcap) if logit_softcap else 0.0
        for k, v in kwargs.items():
            setattr(self, k, v)
        # the names the serving path shares with the other families
        self.hidden_size, self.vocab_size, self.num_hidden_layers = self.width, self.vocab, len(layers)
        self.pad_token_id = self.bos_token_id = self.eos_token_id = None
        self.quantize = None
        for i, lay in enumerate(layers):
            if lay["type"] not in MIXER_TYPES:
                raise ValueError(f"layer {i}: unknown mixer type {lay['type']!r}")
            f = lay.get("mlp")
            if f and f.get("kind") not in ("dense", "moe"):
                raise ValueError(f"layer {i}: unknown feed-forward kind {f.get('kind')!r}")

    @classmethod
    def from_json(cls, path: str) -> "FidatarConfig":
        with open(path) as f:
            return cls(**json.load(f))

    def to_dict(self):
        d = {"architecture": "Fidatar", "width": self.width, "vocab": self.vocab, "layers": self.layers, "norm": {"eps": self.eps},
             "embedding": {"scale": self.embedding_scale}, "postln_alpha": self.postln_alpha}
        if self.logit_softcap:
            d["logit_softcap"] = self.logit_softcap
        return d


class FidatarLayer:
    def __init__(self, i: int, config: FidatarConfig, weights):
        lay = config.layers[i]
        m, p = lay["mixer"], f"l{i}.mix"
        heads, dim = int(m["heads"]), int(m["dim"])
        vdim = int(m.get("vdim", dim))
        if lay["type"] == "attention":
            mask, rot = m.get("mask") or {}, m.get("rot") or {}
            self.mixer = HalfRotatedBlockAttention(
                weights, p, i, heads=heads, kv_heads=int(m.get("kv_heads", heads)), dim=dim, vdim=vdim, scale=float(m["scale"]), eps=config.eps,
                chunk=int(mask.get("size", 0)), rot_base=float(rot.get("base", 10000.0)), rot_dims=int(rot.get("dims", 0)),
                rot_scaling=rot.get("scaling"))
        else:
            self.mixer = MatrixMemory(weights, p, i, heads=heads, dim=dim, vdim=vdim, gate_cap=float(m["gate_cap"]), eps=config.eps,
                                      read_eps=MEMORY_READ_EPS)
        self.kv_shape, self.state_shape = self.mixer.kv_shape, self.mixer.state_shape
        f = lay.get("mlp")
        self.ff = None
        self.routed = bool(f) and f["kind"] == "moe"
        if self.routed:
            r = f["router"]
            g = r.get("groups") or {}
            count = int(g.get("count", 1))
            self.ff = RoutedExperts(weights, f"l{i}.mlp", experts=int(r["experts"]), top=int(r["top"]), shared=False, weight_on_input=False,
                                    unit="relu2", groups=count, keep_groups=int(g.get("keep", count)), grouped_sigmoid=float(r.get("scale", 1.0)))
        elif f:
            self.ff = ActivatedMLP(weights, f"l{i}.mlp", act="relu2")

    def feed_forward(self, h, routing):
        if self.routed:
            return self.ff(h, defer=True, routed=(*routing, None))
        return self.ff(h, partial=True)


class FlashFidatarModel:
    def __init__(self, config: FidatarConfig, weights):
        if weights.process_group.size() != 1:
            raise NotImplementedError("Fidatar is served by one process per model: its layers are not sharded")
        self.config = config
        self.dtype = weights.dtype
        self.embed = weights.get_tensor("embed").contiguous()
        self.layers = [FidatarLayer(i, config, weights) for i in range(len(config.layers))]
        norms = [f"l{i}.norm{q}" for i, layer in enumerate(self.layers) for q in ((1, 2) if layer.ff is not None else (1,))]
        self.residual = PostNormResidual(weights, norms, "final.norm", config.postln_alpha, config.eps)
        # cache geometry, read by FlashCausalLM
        self.kv_layer_shapes = [l.kv_shape for l in self.layers]
        self.state_layer_shapes = [l.state_shape for l in self.layers]
        shapes = [s for s in self.kv_layer_shapes if s is not None]
        self.num_heads = max(l.mixer.H for l in self.layers)
        self.num_key_value_heads = max([s[0] for s in shapes], default=1)
        self.head_size = max([s[1] for s in shapes], default=8)
        self.supports_ragged_steps = True

    def forward(self, input_ids, position_ids, cu_seqlens_q, max_s, inputs_embeds, kv):
        if inputs_embeds is not None:
            raise NotImplementedError("prompt prefixes (inputs_embeds) are not wired into the fp32-residual path")
        dt, residual, n = self.dtype, self.residual, len(self.layers)
        kv.cu_seqlens_q = cu_seqlens_q
        traced = kv.residual_trace is not None
        # a sublayer's fp32 products of the stream (gates, router logits) come with its input
        x, h, products = residual.begin(input_ids, self.embed, self.config.embedding_scale, dt, self.layers[0].mixer.products)
        q = 0
        for i, layer in enumerate(self.layers):
            last = i + 1 == n
            nxt = None if last else self.layers[i + 1].mixer.products
            y = layer.mixer.forward(h, products, position_ids, kv)
            if layer.ff is not None:
                x, h, products = residual.step(q, x, y, dt, layer.ff.products if layer.routed else None)
                q += 1
                y = layer.feed_forward(h, products)
            x, h, products = residual.step(q, x, y, dt, nxt, last=last, keep_x=traced or not last)
            q += 1
            if traced:
                kv.residual_trace.append(x.clone())
        return h  # final-normed, in the serving dtype

    __call__ = forward


class FlashFidatarForCausalLM:
    def __init__(self, config: FidatarConfig, weights):
        self.config = config
        self.model = FlashFidatarModel(config, weights)
        self.lm_head = FastLinear(weights.get_tensor("head").contiguous(), None)
        self.supports_ragged_steps = True

    def get_input_embeddings(self):
        return None

    @property
    def num_layers(self):
        return len(self.model.layers)

    def forward(self, input_ids, position_ids, cu_seqlens_q, max_s, inputs_embeds=None, kv=None,
                lm_head_indices: Optional[torch.Tensor] = None):
        """fp32 logits [T or len(lm_head_indices), vocab], soft-capped."""
        hidden = self.model(input_ids, position_ids, cu_seqlens_q, max_s, inputs_embeds, kv)
        if lm_head_indices is not None:
            hidden = hidden.index_select(0, lm_head_indices)
        if hidden.shape[0] == 0:
            return torch.empty((0, self.config.vocab), dtype=torch.float32, device=hidden.device)
        # fp32 logits from the weight-streaming kernel's fp32 accumulators, 256 rows at a time (the library GEMM above that size
        # would round them to the serving dtype first)
        if hidden.shape[0] <= 256:
            logits = self.lm_head(hidden, out_f32=True)
        else:
            logits = torch.cat([self.lm_head(hidden[i:i + 256], out_f32=True) for i in range(0, hidden.shape[0], 256)], 0)
        if self.config.logit_softcap:
            native.logit_softcap(logits, self.config.logit_softcap)
        return logits

    __call__ = forward
