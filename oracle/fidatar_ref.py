"""Plain CPU restatement of the Fidatar decoder, one function per mechanism.  TEST INFRASTRUCTURE ONLY: nothing of the serving
path imports this file and it imports nothing of the serving path.

Fidatar norms AFTER the sum: both sublayers of a layer read the stream x itself,
    x <- N(c x + mixer(x)) * w1;    x <- N(c x + ff(x)) * w2          N(z) = z / sqrt(mean z^2 + eps), c one constant of the model
with a scaled embedding in front, one more norm, an untied head and capped logits behind.  Mixers:
  * mlstm      a matrix memory with exponential gates: capped log gates i, f per head, a running maximum m that starts at 0, state
               S and normaliser n scaled by e^-m, a read-out divided by max(|n . q|, e^-m) + 1e-6, per-head norm, sigmoid output gate;
  * attention  GQA with projection biases, gained per-head norms of q and k, half-split partial rotation with YaRN frequencies,
               queries that see only their own block of positions, and a 1 in the softmax denominator.
Feed-forward: W_down relu(W_up h)^2, dense or a mixture of such units chosen by sigmoid scores among the best groups of
neighbours (a group counts by its two best scores); or none.

All arithmetic is in `DT` (float64) on the CPU; weights are taken as stored.  A sequence is processed in any portions through
an explicit per-sequence state (`new_state` / `advance`); `forward` is one portion from an empty state."""
import copy
import math
from typing import Dict, List, Optional

import torch

DT = torch.float64
# what guards the division of the matrix memory's read-out
READ_EPS = 1e-6
# filled by `route` while not None: how far (in score) a token's choice of groups and of experts is from another choice
ROUTER_MARGINS: Optional[list] = None
# filled by `mlstm` while not None: |S^T q| sqrt(dk) / (|S| |q|) per token and head, about one for a q of no particular direction.  The
# read-out is normed, so a q all but orthogonal to what S holds (the first tokens' S has rank one!) turns rounding into direction.
READ_MARGINS: Optional[list] = None


# ---- small pieces ---------------------------------------------------------------------------------------------------------
def rms_unit(z, eps: float):
    return z / torch.sqrt((z * z).mean(-1, keepdim=True) + eps)


def relu2(z):
    return torch.clamp(z, min=0) ** 2


def yarn_frequencies(base: float, dims: int, scaling: Optional[dict] = None):
    """(frequencies of the dims / 2 pairs, factor on cos and sin)."""
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return torch.tensor(plain, dtype=DT), 1.0
    fac, orig = float(scaling["factor"]), float(scaling["original"])
    at = lambda turns: dims * math.log(orig / (2 * math.pi * turns)) / (2 * math.log(base))
    lo = max(math.floor(at(float(scaling["fast"]))), 0)
    hi = min(math.ceil(at(float(scaling["slow"]))), dims - 1)
    out = []
    for i, f in enumerate(plain):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / fac * r + f * (1 - r))
    return torch.tensor(out, dtype=DT), 0.1 * math.log(fac) + 1.0


def turn_halves(x, pos, freq, amp: float = 1.0):
    """x [T, heads, D]: channels (i, i + n), i < n = len(freq), turn by pos * freq[i] and grow by amp; the rest pass."""
    n = len(freq)
    if n == 0:
        return x
    ang = pos.to(DT)[:, None] * freq[None]
    c, s = (amp * torch.cos(ang))[:, None], (amp * torch.sin(ang))[:, None]
    u, v = x[..., :n], x[..., n:2 * n]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * n:]], -1)


def attend_in_blocks(q, K, V, pos, scale: float, block: int = 0):
    """q [T, H, dk] at positions pos; K [n, G, dk], V [n, G, dv] of positions 0 .. n - 1; 1 joins every denominator."""
    T, H, _ = q.shape
    n, G, dv = V.shape
    j = torch.arange(n)
    out = torch.empty(T, H, dv, dtype=DT)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ K[:, g].T) * scale
        seen = j[None] <= pos[:, None]
        if block:
            seen &= (j // block)[None] == (pos // block)[:, None]
        s = torch.where(seen, s, torch.full_like(s, -math.inf))
        m = s.max(-1, keepdim=True).values.clamp(min=0)
        e = torch.exp(s - m)
        out[:, h] = (e / (torch.exp(-m) + e.sum(-1, keepdim=True))) @ V[:, g]
    return out


# ---- mixers ---------------------------------------------------------------------------------------------------------------
def block_attention(h, pos, p, m: dict, eps: float, st: dict):
    T, H = h.shape[0], int(m["heads"])
    G, dk = int(m.get("kv_heads", H)), int(m["dim"])
    dv = int(m.get("vdim", dk))
    q = (h @ p["q"].T + p["q.b"]).view(T, H, dk)
    k = (h @ p["k"].T + p["k.b"]).view(T, G, dk)
    v = (h @ p["v"].T + p["v.b"]).view(T, G, dv)
    q, k = rms_unit(q, eps) * p["q.norm"], rms_unit(k, eps) * p["k.norm"]
    rot = m.get("rot")
    if rot:
        f, amp = yarn_frequencies(float(rot["base"]), int(rot["dims"]), rot.get("scaling"))
        q, k = turn_halves(q, pos, f, amp), turn_halves(k, pos, f, amp)
    st["k"], st["v"] = torch.cat([st["k"], k]), torch.cat([st["v"], v])
    o = attend_in_blocks(q, st["k"], st["v"], pos, float(m["scale"]), int((m.get("mask") or {}).get("size", 0)))
    return o.reshape(T, H * dv) @ p["o"].T


def matrix_memory_step(S, n, mx, q, k, v, i, f):
    """One token: S [H, dk, dv], n [H, dk], mx [H] with gates i, f [H] (logarithms); returns (S, n, mx, read-out [H, dv])."""
    top = torch.maximum(f + mx, i)
    keep, write = torch.exp(f + mx - top), torch.exp(i - top)
    S = keep[:, None, None] * S + write[:, None, None] * k[:, :, None] * v[:, None, :]
    n = keep[:, None] * n + write[:, None] * k
    den = torch.maximum((n * q).sum(-1).abs(), torch.exp(-top)) + READ_EPS
    return S, n, top, (S * q[:, :, None]).sum(1) / den[:, None]


def mlstm(h, p, m: dict, eps: float, st: dict):
    T, H, dk = h.shape[0], int(m["heads"]), int(m["dim"])
    dv, cap = int(m.get("vdim", dk)), float(m["gate_cap"])
    q = (h @ p["q"].T).view(T, H, dk) * dk ** -0.5
    k, v = (h @ p["k"].T).view(T, H, dk), (h @ p["v"].T).view(T, H, dv)
    soft = lambda z: cap * torch.tanh(z / cap)
    i = soft(h @ p["i"].T + p["i.b"])
    f = torch.nn.functional.logsigmoid(soft(h @ p["f"].T + p["f.b"]))
    S, n, mx, rows = st["S"], st["n"], st["m"], []
    for t in range(T):
        S, n, mx, o = matrix_memory_step(S, n, mx, q[t], k[t], v[t], i[t], f[t])
        rows.append(o)
        if READ_MARGINS is not None:
            size = (S * S).sum((1, 2)).sqrt() * (q[t] * q[t]).sum(-1).sqrt()
            READ_MARGINS.extend(((S * q[t][:, :, None]).sum(1).norm(dim=-1) * dk ** 0.5 / size.clamp_min(1e-30)).tolist())
    st["S"], st["n"], st["m"] = S, n, mx
    o = rms_unit(torch.stack(rows), eps).reshape(T, H * dv) * p["norm"]
    return (o * torch.sigmoid(h @ p["g"].T)) @ p["o"].T


# ---- feed-forward ---------------------------------------------------------------------------------------------------------
def unit(h, p, prefix: str = ""):
    return relu2(h @ p[prefix + "up"].T) @ p[prefix + "down"].T


def route(h, w, r: dict):
    """(experts [T, top], weights [T, top])."""
    s = torch.sigmoid(h @ w.T)
    T, E = s.shape
    top, g = int(r["top"]), r.get("groups") or {}
    count = int(g.get("count", 1))
    keep = int(g.get("keep", count))
    allowed = torch.ones(T, E, dtype=torch.bool)
    if keep < count:
        per = E // count
        rank = s.view(T, count, per).topk(min(2, per), dim=-1).values.sum(-1)
        order = rank.sort(-1, descending=True)
        allowed = torch.zeros(T, count, dtype=torch.bool).scatter_(1, order.indices[:, :keep], True).repeat_interleave(per, 1)
        if ROUTER_MARGINS is not None:
            ROUTER_MARGINS.extend((order.values[:, keep - 1] - order.values[:, keep]).tolist())
    c = torch.where(allowed, s, torch.full_like(s, -1.0))
    val, idx = c.topk(top, dim=-1)
    if ROUTER_MARGINS is not None and top < E:
        ROUTER_MARGINS.extend((val[:, -1] - c.topk(top + 1, dim=-1).values[:, -1]).tolist())
    return idx, val * float(r.get("scale", 1.0))


def mixture(h, p, f: dict):
    idx, w = route(h, p["router"], f["router"])
    out = torch.zeros(h.shape[0], p["e0.down"].shape[0], dtype=DT)
    for e in range(int(f["router"]["experts"])):
        hit = (idx == e)
        rows = hit.any(-1)
        if rows.any():
            out[rows] += (w * hit).sum(-1, keepdim=True)[rows] * unit(h[rows], p, f"e{e}.")
    return out


# ---- the model ------------------------------------------------------------------------------------------------------------
class FidatarRef:
    def __init__(self, config: dict, tensors: Dict[str, torch.Tensor]):
        self.c = config
        self.t = {k: v.to(DT) for k, v in tensors.items()}
        self.eps = float(config["norm"]["eps"])
        self.alpha = float(config["postln_alpha"])

    def sub(self, prefix: str) -> Dict[str, torch.Tensor]:
        return {k[len(prefix):]: v for k, v in self.t.items() if k.startswith(prefix)}

    def new_state(self) -> dict:
        layers = []
        for lay in self.c["layers"]:
            m = lay["mixer"]
            H, dk = int(m["heads"]), int(m["dim"])
            dv = int(m.get("vdim", dk))
            if lay["type"] == "attention":
                G = int(m.get("kv_heads", H))
                layers.append({"k": torch.zeros(0, G, dk, dtype=DT), "v": torch.zeros(0, G, dv, dtype=DT)})
            elif lay["type"] == "mlstm":
                layers.append({"S": torch.zeros(H, dk, dv, dtype=DT), "n": torch.zeros(H, dk, dtype=DT), "m": torch.zeros(H, dtype=DT)})
            else:
                raise ValueError(lay["type"])
        return {"layers": layers, "n": 0}

    def layer(self, i: int, x, pos, st: dict):
        lay, t = self.c["layers"][i], self.t
        p = self.sub(f"l{i}.mix.")
        y = block_attention(x, pos, p, lay["mixer"], self.eps, st) if lay["type"] == "attention" else mlstm(x, p, lay["mixer"], self.eps, st)
        x = rms_unit(self.alpha * x + y, self.eps) * t[f"l{i}.norm1"]
        if lay.get("mlp"):
            q = self.sub(f"l{i}.mlp.")
            y = unit(x, q) if lay["mlp"]["kind"] == "dense" else mixture(x, q, lay["mlp"])
            x = rms_unit(self.alpha * x + y, self.eps) * t[f"l{i}.norm2"]
        return x

    def advance(self, state: dict, tokens: List[int], trace: Optional[list] = None) -> torch.Tensor:
        """Feeds the next tokens of a sequence; returns the logits [len(tokens), vocab].  trace: receives the stream after every layer."""
        t, n0 = self.t, state["n"]
        pos = torch.arange(n0, n0 + len(tokens))
        x = t["embed"][torch.tensor(tokens)] * float((self.c.get("embedding") or {}).get("scale", 1.0))
        for i in range(len(self.c["layers"])):
            x = self.layer(i, x, pos, state["layers"][i])
            if trace is not None:
                trace.append(x)
        state["n"] = n0 + len(tokens)
        logits = (rms_unit(x, self.eps) * t["final.norm"]) @ t["head"].T
        cap = self.c.get("logit_softcap")
        return float(cap) * torch.tanh(logits / float(cap)) if cap else logits

    def forward(self, tokens: List[int], trace: Optional[list] = None) -> torch.Tensor:
        return self.advance(self.new_state(), tokens, trace)


def clear_cut_tokens(config: dict, tensors, n: int, seed: int, margin: float = 0.03, read_margin: float = 0.3) -> List[int]:
    """n random tokens, each drawn again until no router of the model is within `margin` (in score) of choosing other experts for it
    and no memory's read-out is below `read_margin` of its usual size: what a reduced-precision run computes for them differs from
    this restatement by rounding, not by a decision."""
    global ROUTER_MARGINS, READ_MARGINS
    g = torch.Generator().manual_seed(seed)
    ref = FidatarRef(config, tensors)
    state, toks = ref.new_state(), []
    try:
        while len(toks) < n:
            best = None
            for _ in range(60):
                t = int(torch.randint(0, config["vocab"], (1,), generator=g))
                trial = copy.deepcopy(state)
                ROUTER_MARGINS, READ_MARGINS = [], []
                ref.advance(trial, [t])
                closest = min(min(ROUTER_MARGINS, default=margin) / margin, min(READ_MARGINS, default=read_margin) / read_margin)
                if best is None or closest > best[0]:
                    best = (closest, t, trial)
                if closest >= 1.0:
                    break
            state = best[2]
            toks.append(best[1])
    finally:
        ROUTER_MARGINS = READ_MARGINS = None
    return toks
