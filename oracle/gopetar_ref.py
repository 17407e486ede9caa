"""Plain CPU restatement of the Gopetar decoder, one function per mechanism.  TEST INFRASTRUCTURE ONLY: nothing of the serving
path imports this file and it imports nothing of the serving path.

Gopetar keeps s residual streams X_1 .. X_s per token instead of one, all equal to the scaled embedding at the start.  A
sublayer f (mixer, then feed-forward) of a layer reads a weighted sum of them and its result is spread over all of them while
they are mixed:
    u = sum_a c_in[a] X_a;    y = f(N(u) g);    X'_b = sum_a M[a, b] X_a + c_out[b] y        N(u) = u / sqrt(mean u^2 + eps), g one number
After the last layer x = sum_a X_a, a final norm of the same kind and an untied head.  Mixers:
  * parallel           left: GQA softmax attention with projection biases, partial interleaved rotation with piecewise scaled
                       frequencies, values that are rotated by their position and turned back by the reader's, capped scores, a
                       sliding window and a sink in the denominator;  right: a gated recurrence S <- (1 - z) S + z c whose gate and
                       candidate read the current token only.  The two results are added with fixed weights;
  * latent_attention   queries and keys / values through normed low-rank latents, no positions; a layer may read the latents
                       another layer cached.
Feed-forward: a softmax-of-the-chosen mixture of clamped gated units plus a shared one behind a sigmoid gate; or none.

All arithmetic is in `DT` (float64) on the CPU; weights are taken as stored.  A sequence is processed in any portions through
an explicit per-sequence state (`new_state` / `advance`); `forward` is one portion from an empty state."""
import math
from typing import Dict, List, Optional

import torch

DT = torch.float64
# the slope of the gated unit's sigmoid
GLU_ALPHA = 1.702
# filled by `mixture` while not None: distance between the last chosen and the first unchosen logit, per token
ROUTER_MARGINS: Optional[list] = None


# ---- small pieces ---------------------------------------------------------------------------------------------------------
def rms_unit(z, eps: float):
    return z / torch.sqrt((z * z).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def pair_frequencies(base: float, dims: int, scaling: Optional[dict] = None):
    """base^(-2i / dims), i < dims / 2; with `scaling` wavelengths (2 pi / f) above original / low are divided by `factor`,
    those below original / high kept, and those between blended linearly in original / wavelength."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling:
            wave = 2 * math.pi / f
            lo, hi, orig, fac = (float(scaling[k]) for k in ("low", "high", "original", "factor"))
            if wave > orig / lo:
                f = f / fac
            elif not wave < orig / hi:
                s = (orig / wave - lo) / (hi - lo)
                f = (1 - s) * f / fac + s * f
        out.append(f)
    return torch.tensor(out, dtype=DT)


def turn_pairs(x, pos, freq, sign: float = 1.0):
    """x [T, heads, D]: channels (2i, 2i + 1), i < len(freq), turn by sign * pos * freq[i]; the rest pass."""
    n = len(freq)
    if n == 0:
        return x
    ang = sign * pos.to(DT)[:, None] * freq[None]
    c, s = torch.cos(ang)[:, None], torch.sin(ang)[:, None]
    u, v = x[..., 0:2 * n:2], x[..., 1:2 * n:2]
    out = x.clone()
    out[..., 0:2 * n:2] = u * c - v * s
    out[..., 1:2 * n:2] = v * c + u * s
    return out


def attend(q, K, V, pos, scale: float, window: int = 0, cap: float = 0.0, sink=None):
    """q [T, H, dk] at positions pos; K [n, G, dk], V [n, G, dv] of positions 0 .. n - 1.  Returns [T, H, dv]."""
    T, H, _ = q.shape
    n, G, dv = V.shape
    j = torch.arange(n)
    out = torch.empty(T, H, dv, dtype=DT)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ K[:, g].T) * scale
        if cap:
            s = cap * torch.tanh(s / cap)
        d = pos[:, None] - j[None]
        seen = d >= 0
        if window:
            seen &= d < window
        s = torch.where(seen, s, torch.full_like(s, -math.inf))
        m = s.max(-1, keepdim=True).values
        if sink is not None:
            m = torch.maximum(m, sink[h])
        e = torch.exp(s - m)
        den = e.sum(-1, keepdim=True)
        if sink is not None:
            den = den + torch.exp(sink[h] - m)
        out[:, h] = (e / den) @ V[:, g]
    return out


# ---- mixers ---------------------------------------------------------------------------------------------------------------
def rotated_value_attention(h, pos, p, m: dict, st: dict):
    T, H = h.shape[0], int(m["heads"])
    G, dk = int(m.get("kv_heads", H)), int(m["dim"])
    dv = int(m.get("vdim", dk))
    proj = lambda n: h @ p[n].T + p.get(n + ".b", torch.zeros(p[n].shape[0], dtype=DT))
    q, k, v = proj("q").view(T, H, dk), proj("k").view(T, G, dk), proj("v").view(T, G, dv)
    rot = m.get("rot")
    if rot:
        f = pair_frequencies(float(rot["base"]), int(rot["dims"]), rot.get("scaling"))
        fv = pair_frequencies(float(rot["base"]), dv)
        q, k, v = turn_pairs(q, pos, f), turn_pairs(k, pos, f), turn_pairs(v, pos, fv)
    st["k"], st["v"] = torch.cat([st["k"], k]), torch.cat([st["v"], v])
    o = attend(q, st["k"], st["v"], pos, float(m["scale"]), int((m.get("mask") or {}).get("size", 0)), float(m.get("softcap") or 0.0), p.get("sink"))
    if rot:
        o = turn_pairs(o, pos, fv, -1.0)
    return o.reshape(T, H * dv) @ p["o"].T


def min_gru(h, p, st: dict):
    z = torch.sigmoid(h @ p["z"].T + p["z.b"])
    u = h @ p["x"].T + p["x.b"]
    cand = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    S, rows = st["S"], []
    for t in range(h.shape[0]):
        S = (1 - z[t]) * S + z[t] * cand[t]
        rows.append(S)
    st["S"] = S
    return (torch.stack(rows) * silu(h @ p["g"].T)) @ p["o"].T


def side_by_side(h, pos, p, m: dict, st: dict):
    part = lambda s: {k[len(s):]: v for k, v in p.items() if k.startswith(s)}
    return float(m["left_scale"]) * rotated_value_attention(h, pos, part("left."), m["left"], st["left"]) + \
        float(m["right_scale"]) * min_gru(h, part("right."), st["right"])


def latent_attention(h, pos, p, m: dict, eps: float, own: dict, source: dict):
    """own: this layer's latents (advanced when it makes its own); source: the latents it attends to."""
    T, H, dk, dv = h.shape[0], int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = ((rms_unit(h @ p["dq"].T, eps) * p["dq.norm"]) @ p["uq"].T).view(T, H, dk)
    if "dkv" in p:
        own["c"] = torch.cat([own["c"], rms_unit(h @ p["dkv"].T, eps) * p["dkv.norm"]])
    c = source["c"]
    K, V = (c @ p["uk"].T).view(-1, H, dk), (c @ p["uv"].T).view(-1, H, dv)
    return attend(q, K, V, pos, float(m["scale"])).reshape(T, H * dv) @ p["o"].T


# ---- feed-forward ---------------------------------------------------------------------------------------------------------
def clamped_unit(h, p, prefix: str, limit: float):
    g = torch.clamp(h @ p[prefix + "gate"].T, max=limit)
    u = torch.clamp(h @ p[prefix + "up"].T, -limit, limit)
    return (g * torch.sigmoid(GLU_ALPHA * g) * (u + 1)) @ p[prefix + "down"].T


def route(h, w, top: int):
    z = h @ w.T
    val, idx = z.topk(top, dim=-1)
    if ROUTER_MARGINS is not None and top < z.shape[-1]:
        ROUTER_MARGINS.extend((val[:, -1] - z.topk(top + 1, dim=-1).values[:, -1]).tolist())
    return idx, torch.softmax(val, -1)


def mixture(h, p, f: dict):
    idx, w = route(h, p["router"], int(f["router"]["top"]))
    out = torch.zeros(h.shape[0], p["e0.down"].shape[0], dtype=DT)
    for e in range(int(f["router"]["experts"])):
        hit = (idx == e)
        rows = hit.any(-1)
        if rows.any():
            out[rows] += (w * hit).sum(-1, keepdim=True)[rows] * clamped_unit(h[rows], p, f"e{e}.", float(f["expert"]["limit"]))
    if f.get("shared"):
        out = out + torch.sigmoid(h @ p["shared.sg"].reshape(1, -1).T) * clamped_unit(h, p, "shared.", float(f["shared"]["limit"]))
    return out


# ---- the model ------------------------------------------------------------------------------------------------------------
def hyper_sublayer(X, t, prefix: str, gain, eps: float, f):
    """X [T, s, W]; the three weights of the connection are `<prefix>.in` [s], `.mix` [s, s] (from, to) and `.out` [s]."""
    u = torch.einsum("s,tsw->tw", t[prefix + ".in"], X)
    y = f(rms_unit(u, eps) * gain)
    return torch.einsum("sb,tsw->tbw", t[prefix + ".mix"], X) + t[prefix + ".out"][None, :, None] * y[:, None]


class GopetarRef:
    def __init__(self, config: dict, tensors: Dict[str, torch.Tensor]):
        self.c = config
        self.t = {k: v.to(DT) for k, v in tensors.items()}
        self.eps = float(config["norm"]["eps"])

    def sub(self, prefix: str) -> Dict[str, torch.Tensor]:
        return {k[len(prefix):]: v for k, v in self.t.items() if k.startswith(prefix)}

    def new_state(self) -> dict:
        layers = []
        for lay in self.c["layers"]:
            m = lay["mixer"]
            if lay["type"] == "parallel":
                l = m["left"]
                G = int(l.get("kv_heads", l["heads"]))
                layers.append({"left": {"k": torch.zeros(0, G, int(l["dim"]), dtype=DT), "v": torch.zeros(0, G, int(l.get("vdim", l["dim"])), dtype=DT)},
                               "right": {"S": torch.zeros(int(m["right"]["width"]), dtype=DT)}})
            elif lay["type"] == "latent_attention":
                layers.append({"c": torch.zeros(0, int(m["kv_rank"]), dtype=DT)})
            else:
                raise ValueError(lay["type"])
        return {"layers": layers, "n": 0}

    def layer(self, i: int, X, pos, layers: List[dict]):
        lay, t, eps = self.c["layers"][i], self.t, self.eps
        m, p = lay["mixer"], self.sub(f"l{i}.mix.")
        if lay["type"] == "parallel":
            mixer = lambda h: side_by_side(h, pos, p, m, layers[i])
        else:
            mixer = lambda h: latent_attention(h, pos, p, m, eps, layers[i], layers[i if m.get("kv_from") is None else int(m["kv_from"])])
        X = hyper_sublayer(X, t, f"l{i}.hc1", t[f"l{i}.norm1"], eps, mixer)
        if lay.get("mlp"):
            q = self.sub(f"l{i}.mlp.")
            X = hyper_sublayer(X, t, f"l{i}.hc2", t[f"l{i}.norm2"], eps, lambda h: mixture(h, q, lay["mlp"]))
        return X

    def advance(self, state: dict, tokens: List[int], trace: Optional[list] = None) -> torch.Tensor:
        """Feeds the next tokens of a sequence; returns the logits [len(tokens), vocab].  trace: receives the sum of the streams
        after every layer."""
        t, n0 = self.t, state["n"]
        pos = torch.arange(n0, n0 + len(tokens))
        x = t["embed"][torch.tensor(tokens)] * float((self.c.get("embedding") or {}).get("scale", 1.0))
        X = x[:, None].repeat(1, int(self.c["streams"]), 1)
        for i in range(len(self.c["layers"])):
            X = self.layer(i, X, pos, state["layers"])
            if trace is not None:
                trace.append(X.sum(1))
        state["n"] = n0 + len(tokens)
        return (rms_unit(X.sum(1), self.eps) * t["final.norm"]) @ t["head"].T

    def forward(self, tokens: List[int], trace: Optional[list] = None) -> torch.Tensor:
        return self.advance(self.new_state(), tokens, trace)


def clear_cut_tokens(config: dict, tensors, n: int, seed: int, margin: float = 0.15) -> List[int]:
    """n random tokens, each drawn again until no router of the model is within `margin` (in logit) of choosing other experts
    for it: what a reduced-precision run computes for them differs from this restatement by rounding, not by a decision."""
    import copy

    global ROUTER_MARGINS
    g = torch.Generator().manual_seed(seed)
    ref = GopetarRef(config, tensors)
    state, toks = ref.new_state(), []
    try:
        while len(toks) < n:
            best = None
            for _ in range(60):
                t = int(torch.randint(0, config["vocab"], (1,), generator=g))
                trial = copy.deepcopy(state)
                ROUTER_MARGINS = []
                ref.advance(trial, [t])
                closest = min(ROUTER_MARGINS, default=margin)
                if best is None or closest > best[0]:
                    best = (closest, t, trial)
                if closest >= margin:
                    break
            state = best[2]
            toks.append(best[1])
    finally:
        ROUTER_MARGINS = None
    return toks
