"""Gopetar: a decoder with several fp32 residual streams X_1 .. X_s per token, all equal to the scaled embedding at the start.
Every sublayer f — a layer's mixer, then its feed-forward — reads a weighted sum of the streams and is spread over all of them
while they are mixed:

    u = sum_a in[a] X_a;    X_b <- sum_a mix[a, b] X_a + out[b] f(N(u) g)          N(u) = u / sqrt(mean u^2 + eps), g one number

and the end of the stack reads the plain sum.  Mixers: `parallel` (GQA softmax attention with scaled partial rotation, rotated
values, capped scores, a sliding window and a sink, beside a minGRU recurrence; the results added with fixed weights) and
`latent_attention` (low-rank query and key / value latents without positions; a layer may read the latents another one cached).
The feed-forward is a mixture of clamped gated units weighted by the softmax over the chosen logits, with a shared unit behind
a sigmoid gate.  Untied head.

config.json gives `width`, `vocab`, `streams`, `norm.eps`, `embedding.scale` and `layers[i].type|mixer|mlp`; tensors are named
`embed`, `l<i>.norm1|norm2`, `l<i>.hc1|hc2.in|out|mix`, `l<i>.mix.*`, `l<i>.mlp.*`, `final.norm`, `head`.  This file only maps
those keys and names onto the mechanisms of utils/mixers.py; the step (ragged: portions of prompts beside decoded tokens), the
paged KV pool and the recurrent state slots are FlashCausalLM's (models/flash_causal_lm.py)."""
import json
from typing import List, Optional

import torch

from tgis_amd import native
from tgis_amd.utils.layers import FastLinear
from tgis_amd.utils.mixers import HyperStreams, LatentAttention, MinGRU, RoutedExperts, SideBySideMixers, WindowSinkAttention

MIXER_TYPES = ("parallel", "latent_attention")
# the slope of the gated unit's sigmoid: a constant of the design
GLU_ALPHA = 1.702


class GopetarConfig:
    model_type = "gopetar"

    def __init__(self, width: int, vocab: int, layers: List[dict], norm: dict, streams: int = 1, embedding: Optional[dict] = None, **kwargs):
        self.width, self.vocab, self.layers, self.streams = int(width), int(vocab), layers, int(streams)
        self.eps = float(norm["eps"])
        self.embedding_scale = float((embedding or {}).get("scale", 1.0))
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
            if f and f.get("kind") != "moe":
                raise ValueError(f"layer {i}: unknown feed-forward kind {f.get('kind')!r}")
            src = lay["mixer"].get("kv_from")
            if src is not None:
                ok = lay["type"] == "latent_attention" and 0 <= src < i and layers[src]["type"] == "latent_attention" and \
                    layers[src]["mixer"].get("kv_from") is None and layers[src]["mixer"]["kv_rank"] == lay["mixer"]["kv_rank"]
                if not ok:
                    raise ValueError(f"layer {i}: kv_from must name an earlier latent attention layer with latents of its own, of the same rank")

    @classmethod
    def from_json(cls, path: str) -> "GopetarConfig":
        with open(path) as f:
            return cls(**json.load(f))

    def to_dict(self):
        return {"architecture": "Gopetar", "width": self.width, "vocab": self.vocab, "layers": self.layers, "norm": {"eps": self.eps},
                "embedding": {"scale": self.embedding_scale}, "streams": self.streams}


class GopetarLayer:
    def __init__(self, i: int, config: GopetarConfig, weights):
        lay = config.layers[i]
        m, p = lay["mixer"], f"l{i}.mix"
        self.layer_id, self.kind = i, lay["type"]
        self.kv_shape = self.state_shape = None
        if self.kind == "parallel":
            l = m["left"]
            heads, dim = int(l["heads"]), int(l["dim"])
            mask, rot = l.get("mask") or {}, l.get("rot") or {}
            attention = WindowSinkAttention(
                weights, f"{p}.left", i, heads=heads, kv_heads=int(l.get("kv_heads", heads)), dim=dim, vdim=int(l.get("vdim", dim)),
                scale=float(l["scale"]), window=int(mask.get("size", 0)), rot_base=float(rot.get("base", 10000.0)),
                rot_dims=int(rot.get("dims", 0)), rot_scaling=rot.get("scaling"), softcap=float(l.get("softcap") or 0.0),
                turned_values=bool(rot))
            recurrence = MinGRU(weights, f"{p}.right", i, width=int(m["right"]["width"]))
            self.mixer = SideBySideMixers(weights, [attention, recurrence], [float(m.get("left_scale", 1.0)), float(m.get("right_scale", 1.0))])
            self.heads = attention.H
            self.kv_shape, self.state_shape = attention.kv_shape, recurrence.state_shape
        else:
            self.mixer = LatentAttention(weights, p, i, heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=0, vdim=int(m["vdim"]),
                                         kv_rank=int(m["kv_rank"]), scale=float(m["scale"]), eps=config.eps, kv_source=m.get("kv_from"))
            self.heads = self.mixer.H
            self.kv_shape = self.mixer.kv_shape
        f = lay.get("mlp")
        self.ff = None
        if f:
            shared = f.get("shared")
            self.ff = RoutedExperts(weights, f"l{i}.mlp", experts=int(f["router"]["experts"]), top=int(f["router"]["top"]), shared=bool(shared),
                                    softmax_top=True, weight_on_input=False, clamp=(GLU_ALPHA, float(f["expert"]["limit"])),
                                    shared_clamp=(GLU_ALPHA, float(shared["limit"])) if shared else None)

    def mix(self, h, position_ids, kv):
        y = self.mixer.forward(h, position_ids, kv)
        return y[0] if self.kind == "parallel" else y


class FlashGopetarModel:
    def __init__(self, config: GopetarConfig, weights):
        if weights.process_group.size() != 1:
            raise NotImplementedError("Gopetar is served by one process per model: its layers are not sharded")
        self.config = config
        self.dtype = weights.dtype
        self.embed = weights.get_tensor("embed").contiguous()
        self.layers = [GopetarLayer(i, config, weights) for i in range(len(config.layers))]
        # the sublayers in execution order, then the read-out at the end of the stack
        subs = []
        for i, layer in enumerate(self.layers):
            for q in (1, 2) if layer.ff is not None else (1,):
                prefix = f"l{i}.hc{q}"
                subs.append((prefix if weights.has(prefix + ".in") else None, f"l{i}.norm{q}"))
        if config.streams > 1 and any(p is None for p, _ in subs):
            raise ValueError("a sublayer has no connection weights")
        self.residual = HyperStreams(weights, config.streams, subs + [(None, "final.norm")], config.eps, self.embed.device)
        # cache geometry, read by FlashCausalLM (layers that read another layer's latents have none)
        self.kv_layer_shapes = [l.kv_shape for l in self.layers]
        self.state_layer_shapes = [l.state_shape for l in self.layers]
        shapes = [s for s in self.kv_layer_shapes if s is not None]
        self.num_heads = max(l.heads for l in self.layers)
        self.num_key_value_heads = max(s[0] for s in shapes)
        self.head_size = max(s[1] for s in shapes)
        self.supports_ragged_steps = True

    def forward(self, input_ids, position_ids, cu_seqlens_q, max_s, inputs_embeds, kv):
        if inputs_embeds is not None:
            raise NotImplementedError("prompt prefixes (inputs_embeds) are not wired into the fp32-residual path")
        dt, residual = self.dtype, self.residual
        kv.cu_seqlens_q = cu_seqlens_q
        X, h = residual.begin(input_ids, self.embed, self.config.embedding_scale, dt)
        q = 0
        for layer in self.layers:
            # the mixture's router rides in the update in front of it, its sum in the update behind it
            router = layer.ff.plain_router if layer.ff is not None else None
            X, h, routed = residual.step(q, X, layer.mix(h, position_ids, kv), dt, router)
            q += 1
            if layer.ff is not None:
                X, h, _ = residual.step(q, X, layer.ff(h, defer=True, routed=routed), dt)
                q += 1
            if kv.residual_trace is not None:
                kv.residual_trace.append(X.sum(1))
        return h  # final-normed, in the serving dtype

    __call__ = forward


class FlashGopetarForCausalLM:
    def __init__(self, config: GopetarConfig, weights):
        self.config = config
        self.model = FlashGopetarModel(config, weights)
        self.lm_head = FastLinear(weights.get_tensor("head").contiguous(), None)
        self.supports_ragged_steps = True

    def get_input_embeddings(self):
        return None

    @property
    def num_layers(self):
        return len(self.model.layers)

    def forward(self, input_ids, position_ids, cu_seqlens_q, max_s, inputs_embeds=None, kv=None,
                lm_head_indices: Optional[torch.Tensor] = None):
        """fp32 logits [T or len(lm_head_indices), vocab]."""
        hidden = self.model(input_ids, position_ids, cu_seqlens_q, max_s, inputs_embeds, kv)
        if lm_head_indices is not None:
            hidden = hidden.index_select(0, lm_head_indices)
        if hidden.shape[0] == 0:
            return torch.empty((0, self.config.vocab), dtype=torch.float32, device=hidden.device)
        # fp32 logits from the weight-streaming kernel's fp32 accumulators, 256 rows at a time (the library GEMM above that
        # size would round them to the serving dtype first)
        if hidden.shape[0] <= 256:
            return self.lm_head(hidden, out_f32=True)
        return torch.cat([self.lm_head(hidden[i:i + 256], out_f32=True) for i in range(0, hidden.shape[0], 256)], 0)

    __call__ = forward
