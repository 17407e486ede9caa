"""Seeded small Fidatar checkpoints for tests: a config dict and a {name: tensor} dict in the family's tensor naming.
Sizes are arguments; nothing here equals a published model.  TEST INFRASTRUCTURE ONLY."""
from typing import Dict, List, Optional

import torch

SCALING = {"factor": 4.0, "original": 300, "fast": 20.0, "slow": 1.5}


def attention_layer(heads=6, kv_heads=3, dim=32, vdim=24, scale=0.25, chunk: Optional[int] = 40, rot_dims: Optional[int] = 16, rot_base=5000.0,
                    scaling=SCALING, mlp=None) -> dict:
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk:
        m["mask"] = {"size": chunk}
    if rot_dims is not None:
        m["rot"] = {"base": rot_base, "dims": rot_dims}
        if scaling:
            m["rot"]["scaling"] = dict(scaling)
    return {"type": "attention", "mixer": m, "mlp": mlp}


def mlstm_layer(heads=3, dim=24, vdim=40, gate_cap=7.0, mlp=None) -> dict:
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}, "mlp": mlp}


def dense_mlp(ff=88) -> dict:
    return {"kind": "dense", "ff": ff}


def moe_mlp(experts=6, top=2, ff=40, groups: Optional[tuple] = (3, 2), scale=1.8) -> dict:
    r = {"experts": experts, "top": top, "scale": scale}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def make_config(layers: List[dict], width=72, vocab=112, eps=1e-5, scale=2.5, alpha=1.7, softcap: Optional[float] = 9.0) -> dict:
    c = {"architecture": "Fidatar", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps}, "embedding": {"scale": scale},
         "postln_alpha": alpha}
    if softcap:
        c["logit_softcap"] = softcap
    return c


def make_tensors(config: dict, seed: int = 0, dtype=torch.bfloat16) -> Dict[str, torch.Tensor]:
    """N(0, 1 / fan_in) projections (wider for what feeds a softmax, a router or a gate), norm gains around one, forget gates that keep
    for tens of tokens, input gates of either sign, keys and queries of a memory that have something in common.  Values are rounded to `dtype` (what a checkpoint stores)."""
    g = torch.Generator().manual_seed(seed)
    W = config["width"]
    t: Dict[str, torch.Tensor] = {}

    def lin(name, n, k, gain=1.0):
        t[name] = torch.randn(n, k, generator=g) * gain * k ** -0.5

    def vec(name, n, mean=0.0, std=0.1):
        t[name] = mean + torch.randn(n, generator=g) * std

    t["embed"] = torch.randn(config["vocab"], W, generator=g)
    for i, lay in enumerate(config["layers"]):
        m, p = lay["mixer"], f"l{i}.mix"
        H, dk = m["heads"], m["dim"]
        dv = m.get("vdim", dk)
        vec(f"l{i}.norm1", W, 1.0, 0.2)
        if lay["type"] == "attention":
            G = m.get("kv_heads", H)
            for n, rows in (("q", H * dk), ("k", G * dk), ("v", G * dv)):
                lin(f"{p}.{n}", rows, W, 1.5)
                vec(f"{p}.{n}.b", rows, 0.0, 0.3)
            vec(f"{p}.q.norm", dk, 1.2, 0.3)
            vec(f"{p}.k.norm", dk, 1.2, 0.3)
        else:
            for n, rows in (("q", H * dk), ("k", H * dk), ("v", H * dv), ("g", H * dv)):
                lin(f"{p}.{n}", rows, W, 1.3)
            t[f"{p}.k"] = 0.7 * t[f"{p}.q"] + 0.7 * t[f"{p}.k"]  # a token's query asks for keys like its own
            vec(f"{p}.norm", H * dv, 1.0, 0.2)
            lin(f"{p}.i", H, W, 2.0)
            vec(f"{p}.i.b", H, -1.0, 1.5)
            lin(f"{p}.f", H, W, 1.5)
            vec(f"{p}.f.b", H, 3.0, 1.0)
        lin(f"{p}.o", W, H * dv, 1.5)
        f = lay.get("mlp")
        if f:
            vec(f"l{i}.norm2", W, 1.0, 0.2)
            q = f"l{i}.mlp"
            dense = f["kind"] == "dense"
            units = [(q, f["ff"])] if dense else [(f"{q}.e{e}", f["expert"]["ff"]) for e in range(f["router"]["experts"])]
            for name, ff in units:
                lin(f"{name}.up", ff, W, 1.3)
                lin(f"{name}.down", W, ff, 1.3)
            if not dense:
                lin(f"{q}.router", f["router"]["experts"], W, 2.0)
    vec("final.norm", W, 1.0, 0.2)
    lin("head", config["vocab"], W, 3.0)
    return {k: v.to(dtype) for k, v in t.items()}


def standard_layers() -> List[dict]:
    """Both mixers first and last of a pair, every kind of feed-forward, a layer without one, GQA and MHA, blocks and plain causal,
    full and partial rotation, scaled frequencies and plain ones, groups and none."""
    return [mlstm_layer(mlp=moe_mlp()),
            attention_layer(mlp=dense_mlp()),
            mlstm_layer(heads=2, dim=40, vdim=16, gate_cap=15.0, mlp=None),
            attention_layer(heads=4, kv_heads=4, dim=16, vdim=32, chunk=None, rot_dims=16, scaling=None, mlp=moe_mlp(experts=8, top=3, ff=32, groups=(2, 1), scale=0.7)),
            mlstm_layer(heads=4, dim=16, vdim=24, mlp=moe_mlp(experts=4, top=1, ff=56, groups=None, scale=1.0))]


def random_config(seed: int) -> dict:
    """A configuration drawn from the design's whole space: 2 .. 5 layers of any kinds in any order, a feed-forward of either kind or
    none, widths that need not be multiples of 8."""
    import random

    rnd = random.Random(seed)
    pick = rnd.choice

    def mlp():
        kind = rnd.random()
        if kind < 0.2:
            return None
        if kind < 0.5:
            return dense_mlp(ff=pick([16, 33, 64, 130]))
        per, count = pick([1, 2, 3, 5]), pick([1, 2, 4])
        keep = rnd.randint(1, count)
        return moe_mlp(experts=per * count, top=rnd.randint(1, min(per * keep, 5)), ff=pick([16, 20, 40]), groups=(count, keep) if count > 1 or rnd.random() < 0.5 else None,
                       scale=pick([0.5, 1.0, 2.5]))

    def one():
        if rnd.random() < 0.5:
            return mlstm_layer(heads=pick([1, 2, 3, 5]), dim=pick([4, 8, 20, 32, 48, 64]), vdim=pick([8, 12, 32, 40, 96]), gate_cap=pick([2.0, 8.0, 20.0]), mlp=mlp())
        G, dk = pick([1, 2, 3]), pick([8, 16, 24, 32, 64])
        return attention_layer(heads=G * pick([1, 2, 3, 4]), kv_heads=G, dim=dk, vdim=pick([8, 16, 32, 48, 64]), scale=pick([0.1, 0.25, dk ** -0.5]),
                               chunk=pick([None, 1, 7, 32, 50, 64, 100]), rot_dims=pick([None, 0, 2, dk // 2, dk]), rot_base=pick([100.0, 10000.0, 500000.0]),
                               scaling=pick([None, SCALING, {"factor": 16.0, "original": 1000, "fast": 32.0, "slow": 1.0}]), mlp=mlp())

    return make_config([one() for _ in range(rnd.randint(2, 5))], width=pick([24, 36, 40, 64, 100]), vocab=pick([31, 64, 97]), eps=pick([1e-5, 1e-6]),
                       scale=pick([0.5, 1.0, 8.0]), alpha=pick([1.0, 1.5, 4.0]), softcap=pick([None, 5.0, 30.0]))
