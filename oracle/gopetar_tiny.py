"""Seeded small Gopetar checkpoints for tests: a config dict and a {name: tensor} dict in the family's tensor naming.
Sizes are arguments; nothing here equals a published model.  TEST INFRASTRUCTURE ONLY."""
from typing import Dict, List, Optional

import torch

SCALING = {"factor": 3.0, "low": 1.0, "high": 5.0, "original": 200}


def attention_part(heads=6, kv_heads=3, dim=32, vdim=24, scale=0.3, window: Optional[int] = 40, rot_dims=16, rot_base=5000.0, scaling=SCALING,
                   softcap: Optional[float] = 6.0) -> dict:
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if window:
        m["mask"] = {"size": window}
    if rot_dims is not None:
        m["rot"] = {"base": rot_base, "dims": rot_dims}
        if scaling:
            m["rot"]["scaling"] = dict(scaling)
    if softcap:
        m["softcap"] = softcap
    return m


def pair_layer(left: Optional[dict] = None, width=88, left_scale=0.7, right_scale=1.3, mlp=None) -> dict:
    return {"type": "parallel", "mixer": {"left": left or attention_part(), "left_scale": left_scale, "right": {"width": width},
                                          "right_scale": right_scale}, "mlp": mlp}


def latent_layer(heads=3, dim=24, vdim=40, kv_rank=48, q_rank=56, scale=0.2, kv_from: Optional[int] = None, mlp=None) -> dict:
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def moe_mlp(experts=6, top=2, ff=40, limit=0.9, shared_ff: Optional[int] = 56, shared_limit=1.7) -> dict:
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if shared_ff:
        m["shared"] = {"ff": shared_ff, "limit": shared_limit}
    return m


def make_config(layers: List[dict], width=72, vocab=112, eps=1e-5, streams=3, scale=2.5) -> dict:
    return {"architecture": "Gopetar", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps}, "streams": streams,
            "embedding": {"scale": scale}}


def make_tensors(config: dict, seed: int = 0, dtype=torch.bfloat16) -> Dict[str, torch.Tensor]:
    """N(0, 1 / fan_in) projections (wider for what feeds a softmax, a router or a gate), norm gains around one, mixing matrices near
    the identity, sinks of the size of a score.  Values are rounded to `dtype` (what a checkpoint stores)."""
    g = torch.Generator().manual_seed(seed)
    W, s = config["width"], config["streams"]
    t: Dict[str, torch.Tensor] = {}

    def lin(name, n, k, gain=1.0):
        t[name] = torch.randn(n, k, generator=g) * gain * k ** -0.5

    def vec(name, n, mean=0.0, std=0.1):
        t[name] = mean + torch.randn(n, generator=g) * std

    def connection(prefix):
        vec(f"{prefix}.in", s, 0.6, 0.4)
        vec(f"{prefix}.out", s, 1.0, 0.5)
        t[f"{prefix}.mix"] = torch.eye(s) * 0.8 + torch.randn(s, s, generator=g) * 0.15

    t["embed"] = torch.randn(config["vocab"], W, generator=g)
    for i, lay in enumerate(config["layers"]):
        m, p = lay["mixer"], f"l{i}.mix"
        t[f"l{i}.norm1"] = 1.0 + 0.2 * torch.randn((), generator=g)
        connection(f"l{i}.hc1")
        if lay["type"] == "parallel":
            a, q = m["left"], f"{p}.left"
            H, dk = a["heads"], a["dim"]
            G, dv = a.get("kv_heads", H), a.get("vdim", dk)
            for n_, rows, gain in (("q", H * dk, 1.5), ("k", G * dk, 1.5), ("v", G * dv, 1.0)):
                lin(f"{q}.{n_}", rows, W, gain)
                vec(f"{q}.{n_}.b", rows, 0.0, 0.3)
            vec(f"{q}.sink", H, 1.0, 1.5)
            lin(f"{q}.o", W, H * dv, 1.5)
            D, q = m["right"]["width"], f"{p}.right"
            lin(f"{q}.z", D, W, 1.5)
            vec(f"{q}.z.b", D, -1.5, 1.5)
            lin(f"{q}.x", D, W, 1.5)
            vec(f"{q}.x.b", D, 0.0, 0.5)
            lin(f"{q}.g", D, W, 1.5)
            lin(f"{q}.o", W, D)
        else:
            H, dk, dv, rk, rq = m["heads"], m["dim"], m["vdim"], m["kv_rank"], m["q_rank"]
            lin(f"{p}.dq", rq, W)
            vec(f"{p}.dq.norm", rq, 1.0)
            lin(f"{p}.uq", H * dk, rq, 1.5)
            if m.get("kv_from") is None:
                lin(f"{p}.dkv", rk, W)
                vec(f"{p}.dkv.norm", rk, 1.0)
            lin(f"{p}.uk", H * dk, rk, 1.5)
            lin(f"{p}.uv", H * dv, rk, 1.5)
            lin(f"{p}.o", W, H * dv, 1.5)
        f = lay.get("mlp")
        if f:
            q, E, ff = f"l{i}.mlp", f["router"]["experts"], f["expert"]["ff"]
            t[f"l{i}.norm2"] = 1.0 + 0.2 * torch.randn((), generator=g)
            connection(f"l{i}.hc2")
            units = [(f"{q}.e{e}", ff) for e in range(E)] + ([(f"{q}.shared", f["shared"]["ff"])] if f.get("shared") else [])
            for name, n_ in units:
                lin(f"{name}.gate", n_, W, 1.5)
                lin(f"{name}.up", n_, W, 1.5)
                lin(f"{name}.down", W, n_, 1.5)
            lin(f"{q}.router", E, W, 1.5)
            if f.get("shared"):
                lin(f"{q}.shared.sg", 1, W, 2.0)
    t["final.norm"] = 1.0 + 0.2 * torch.randn((), generator=g)
    lin("head", config["vocab"], W)
    return {k: v.to(dtype) for k, v in t.items()}


def standard_layers() -> List[dict]:
    """Both mixers, a layer that reads another one's latents (with sizes of its own otherwise), a layer without a feed-forward,
    GQA and MHA, a window and none, full and partial rotation, scaled frequencies and plain ones, no cap, no shared expert."""
    return [latent_layer(mlp=moe_mlp()),
            pair_layer(mlp=moe_mlp(experts=4, top=1, ff=56, shared_ff=None)),
            latent_layer(heads=4, dim=16, vdim=24, q_rank=40, scale=0.3, kv_from=0, mlp=None),
            pair_layer(left=attention_part(heads=4, kv_heads=4, dim=16, vdim=16, window=None, rot_dims=16, scaling=None, softcap=None), width=60,
                       mlp=moe_mlp(experts=8, top=3, ff=32, shared_ff=32)),
            latent_layer(heads=2, dim=40, vdim=16, kv_rank=32, q_rank=24, mlp=moe_mlp(experts=3, top=3))]


def random_config(seed: int) -> dict:
    """A configuration drawn from the design's whole space: 2 .. 5 layers of any kinds in any order, 1 .. 6 streams, a feed-forward
    or none, widths that need not be multiples of 8."""
    import random

    rnd = random.Random(seed)
    pick = rnd.choice

    def mlp():
        if rnd.random() < 0.2:
            return None
        E = pick([1, 2, 5, 12])
        return moe_mlp(experts=E, top=rnd.randint(1, min(E, 5)), ff=pick([16, 20, 40]), limit=pick([0.5, 1.1, 7.0]), shared_ff=pick([None, 24, 50]),
                       shared_limit=pick([0.7, 3.0]))

    def one(sources):
        if rnd.random() < 0.5:
            src = pick(sources) if sources and rnd.random() < 0.5 else None
            rk = src[1] if src else pick([8, 20, 32, 64, 96])
            return latent_layer(heads=pick([1, 2, 3, 5]), dim=pick([8, 12, 32, 40]), vdim=pick([8, 20, 32, 64]), kv_rank=rk, q_rank=pick([6, 16, 40]),
                                scale=pick([0.1, 0.25]), kv_from=src[0] if src else None, mlp=mlp())
        G = pick([1, 2, 3])
        dk = pick([8, 16, 24, 32, 64])
        left = attention_part(heads=G * pick([1, 2, 3, 4]), kv_heads=G, dim=dk, vdim=pick([8, 16, 32, 48, 64]), scale=pick([0.1, 0.25, dk ** -0.5]),
                              window=pick([None, 1, 7, 32, 50, 64, 100]), rot_dims=pick([None, 0, 2, dk // 2, dk]), rot_base=pick([100.0, 10000.0, 500000.0]),
                              scaling=pick([None, SCALING, {"factor": 8.0, "low": 2.0, "high": 4.0, "original": 1000}]), softcap=pick([None, 2.0, 20.0]))
        return pair_layer(left=left, width=pick([20, 33, 64, 130]), left_scale=pick([0.4, 1.0]), right_scale=pick([0.6, 1.0]), mlp=mlp())

    layers, sources = [], []
    for i in range(rnd.randint(2, 5)):
        layers.append(one(sources))
        m = layers[-1]["mixer"]
        if layers[-1]["type"] == "latent_attention" and m.get("kv_from") is None:
            sources.append((i, m["kv_rank"]))
    if all(l["mixer"].get("kv_from") is not None for l in layers):
        layers[0] = latent_layer(mlp=None)
    return make_config(layers, width=pick([24, 36, 40, 64, 100]), vocab=pick([31, 64, 97]), eps=pick([1e-5, 1e-6]), streams=rnd.randint(1, 6),
                       scale=pick([0.5, 1.0, 8.0]))
