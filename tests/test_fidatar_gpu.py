"""GPU: the Fidatar family on the kernels (FlashCausalLM + utils/mixers.py + csrc/post_norm, matrix_memory, attn_varlen, moe) against
the plain float64 restatement in oracle/fidatar_ref.py, on small seeded checkpoints of their own sizes.

float32 serving is compared tightly (it differs from the oracle by accumulation order only); bfloat16 serving against a bound
that scales with bf16 rounding.  Schedules (whole prompts, token by token, portions down to two tokens, mixed batches, pages and
slots that change hands) are compared with the oracle run whole, where only rounding may differ."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import fidatar_ref as ref
from oracle import fidatar_tiny as tiny

pytestmark = pytest.mark.gpu

TOL = {torch.float32: 2e-4, torch.bfloat16: 0.15}
DTYPES = [torch.float32, torch.bfloat16]
D = torch.float64


def build_lm(cfg, tensors, dtype, pages=64, slots=4, tokenizer=None):
    from tgis_amd.inference_engine.synthetic import InferenceEngine
    from tgis_amd.models.custom_modeling.flash_fidatar_modeling import FidatarConfig
    from tgis_amd.models.flash_causal_lm import FlashCausalLM

    eng = InferenceEngine({k: v.clone() for k, v in tensors.items()}, FidatarConfig(**cfg), dtype, None, tokenizer=tokenizer)
    return FlashCausalLM("synthetic", None, "synthetic", dtype, None, engine=eng, kv_cache_pages=pages, state_slots=slots)


def row_errors(got: torch.Tensor, want: torch.Tensor) -> torch.Tensor:
    """Per row: rms of the centred difference over the rms of the centred reference row."""
    got, want = got.double().cpu(), want.double().cpu()
    assert got.shape == want.shape
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    w = want - want.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt().clamp_min(1e-9)


def rel_err(got, want) -> float:
    return float(row_errors(got, want).max())


def close(got, want, dtype) -> bool:
    return rel_err(got, want) <= TOL[dtype]


def max_err(got, want) -> float:
    """Largest difference over the largest reference value."""
    want = want.double().cpu()
    return float((got.double().cpu() - want).abs().max()) / max(float(want.abs().max()), 1e-12)


_PROMPTS = {}


def rand_tokens(n, cfg, tensors, seed):
    """Random tokens for which no router of the checkpoint is near a tie (drawn again until so): a bfloat16 run then differs from
    the float64 restatement by rounding, not by a decision."""
    key = (json.dumps(cfg, sort_keys=True), n, seed)
    if key not in _PROMPTS:
        _PROMPTS[key] = ref.clear_cut_tokens(cfg, tensors, n, seed)
    return _PROMPTS[key]


@pytest.fixture(scope="module")
def std():
    cfg = tiny.make_config(tiny.standard_layers())
    return cfg, tiny.make_tensors(cfg, seed=3)


# ---- whole model -----------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [40, 75, 300, 600])
def test_whole_prompt_matches_oracle_layer_by_layer(gpu_device, std, dtype, n):
    """40 tokens: products of the stream ride in its update; 75: launches of their own, decode-sized GEMMs; 300: the library GEMMs;
    600: the transposing value writers.  All are as long as every block of the configuration or longer."""
    cfg, tensors = std
    lm = build_lm(cfg, tensors, dtype)
    toks = rand_tokens(600, cfg, tensors, 1)[:n]
    want_trace = []
    want = ref.FidatarRef(cfg, tensors).forward(toks, want_trace)
    with lm.context_manager():
        seq, trace = lm.open_sequence(), []
        got = lm.step_sequences([(seq, toks)], residual_trace=trace)
        lm.close_sequence(seq)
    assert len(trace) == len(want_trace) == 5
    for r, (g, w) in enumerate(zip(trace, want_trace)):
        assert max_err(g, w) <= (1e-4 if dtype == torch.float32 else 0.08), r
    assert close(got, want, dtype), rel_err(got, want)


@pytest.mark.parametrize("dtype", DTYPES)
def test_token_by_token_and_portions_equal_whole(gpu_device, std, dtype):
    cfg, tensors = std
    lm = build_lm(cfg, tensors, dtype)
    toks = rand_tokens(150, cfg, tensors, 2)
    want = ref.FidatarRef(cfg, tensors).forward(toks)
    for cuts in ([1] * 150, [2] * 75, [3, 2, 31, 33, 1, 2, 64, 5, 9], [97, 2, 2, 2, 47], [39, 1, 1, 39, 1, 69], [149, 1]):
        with lm.context_manager():
            seq, outs, at = lm.open_sequence(), [], 0
            for c in cuts:
                outs.append(lm.step_sequences([(seq, toks[at:at + c])]))
                at += c
            lm.close_sequence(seq)
        assert close(torch.cat(outs), want, dtype), (cuts[:4], rel_err(torch.cat(outs), want))


@pytest.mark.parametrize("dtype", DTYPES)
def test_mixed_batches_reuse_pages_and_slots(gpu_device, std, dtype):
    """Five requests through a pool of 9 pages and 3 slots: portions of some beside single tokens of others, a request that
    sits steps out, pages and slots handed on to later requests with whatever their last owner left in them."""
    cfg, tensors = std
    lm = build_lm(cfg, tensors, dtype, pages=9, slots=3)
    model = ref.FidatarRef(cfg, tensors)
    prompts = {k: rand_tokens(n, cfg, tensors, 10 + i) for i, (k, n) in enumerate({"a": 70, "b": 33, "c": 96, "d": 45, "e": 64}.items())}
    want = {k: model.forward(v) for k, v in prompts.items()}
    schedule = [[("a", 31), ("b", 2)], [("a", 1), ("b", 30)], [("a", 2), ("b", 1), ("c", 40)], [("a", 36), ("c", 1)], [("c", 23)],
                [("c", 2), ("d", 44)], [("c", 30), ("d", 1), ("e", 3)], [("e", 60)], [("e", 1)]]
    done, live, got = {k: 0 for k in prompts}, {}, {k: [] for k in prompts}
    with lm.context_manager():
        for step in schedule:
            entries = []
            for rid, cnt in step:
                if rid not in live:
                    live[rid] = lm.open_sequence()
                entries.append((live[rid], prompts[rid][done[rid]:done[rid] + cnt]))
            out = lm.step_sequences(entries)
            at = 0
            for rid, cnt in step:
                got[rid].append(out[at:at + cnt])
                at += cnt
                done[rid] += cnt
                if done[rid] == len(prompts[rid]):
                    lm.close_sequence(live.pop(rid))
    assert not live and lm.kv_cache.free_pages == 9 and lm.state_cache.free_slots == 3
    for rid in prompts:
        assert close(torch.cat(got[rid]), want[rid], dtype), (rid, rel_err(torch.cat(got[rid]), want[rid]))


def test_stale_slot_and_pages_do_not_leak(gpu_device, std):
    """Every state tensor and page filled with large numbers before a request starts: a sequence begins from zeros."""
    cfg, tensors = std
    lm = build_lm(cfg, tensors, torch.float32, pages=8, slots=1)
    for t in lm.state_cache.state + lm.state_cache.shift:
        if t is not None:
            t.fill_(37.0)
    for r in range(lm.num_layers):
        if lm.kv_cache.layer_shapes[r] is not None:
            lm.kv_cache.k_pool(r).fill_(19.0)
            lm.kv_cache.v_pool(r).fill_(-23.0)
    toks = rand_tokens(50, cfg, tensors, 4)
    want = ref.FidatarRef(cfg, tensors).forward(toks)
    with lm.context_manager():
        seq = lm.open_sequence()
        got = torch.cat([lm.step_sequences([(seq, toks[:2])]), lm.step_sequences([(seq, toks[2:])])])
        lm.close_sequence(seq)
    assert close(got, want, torch.float32), rel_err(got, want)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(gpu_device, std, dtype):
    """220 single-token steps behind a short prompt: block edges pass under decoded tokens, states are carried all the way."""
    cfg, tensors = std
    lm = build_lm(cfg, tensors, dtype)
    toks = rand_tokens(240, cfg, tensors, 5)
    want = ref.FidatarRef(cfg, tensors).forward(toks)
    with lm.context_manager():
        seq = lm.open_sequence()
        outs = [lm.step_sequences([(seq, toks[:20])])] + [lm.step_sequences([(seq, [t])]) for t in toks[20:]]
        lm.close_sequence(seq)
    assert close(torch.cat(outs), want, dtype), rel_err(torch.cat(outs), want)


# sizes that the standard configuration happens to make equal, one, or a multiple of eight; other layer orders
OTHER_SHAPES = {
    "one_head_each": dict(layers=[tiny.attention_layer(heads=1, kv_heads=1, dim=8, vdim=8, chunk=5, rot_dims=2),
                                  tiny.mlstm_layer(heads=1, dim=8, vdim=8, mlp=tiny.moe_mlp(experts=1, top=1, groups=(1, 1), scale=1.0))],
                          width=40, vocab=50, alpha=1.0, softcap=None, scale=1.0),
    "only_memories": dict(layers=[tiny.mlstm_layer(heads=5, dim=12, vdim=20, gate_cap=3.0, mlp=tiny.moe_mlp(experts=6, top=4, ff=16, groups=(6, 4))),
                                  tiny.mlstm_layer(heads=2, dim=33, vdim=7, mlp=None), tiny.mlstm_layer(heads=3, dim=4, vdim=48, mlp=tiny.dense_mlp(ff=20))],
                          width=36, vocab=41, alpha=2.0, scale=0.5),
    "only_attention": dict(layers=[tiny.attention_layer(heads=2, kv_heads=1, dim=12, vdim=20, chunk=1, rot_dims=4, mlp=None),
                                   tiny.attention_layer(heads=8, kv_heads=4, dim=24, vdim=8, chunk=33, rot_dims=0, mlp=tiny.moe_mlp(experts=9, top=4, ff=24, groups=(3, 2))),
                                   tiny.attention_layer(heads=16, kv_heads=1, dim=16, vdim=32, chunk=64, rot_dims=None, mlp=tiny.dense_mlp(ff=40))],
                           width=24, vocab=33, alpha=5.0, scale=16.0),
    "odd_widths": dict(layers=[tiny.mlstm_layer(heads=3, dim=10, vdim=6, mlp=tiny.moe_mlp(experts=4, top=2, ff=21, groups=(2, 2))),
                               tiny.attention_layer(heads=3, kv_heads=3, dim=10, vdim=6, chunk=64, rot_dims=6, mlp=tiny.dense_mlp(ff=33))],
                       width=37, vocab=41, scale=3.0),
    "wide_heads": dict(layers=[tiny.mlstm_layer(heads=2, dim=128, vdim=128, mlp=tiny.moe_mlp(experts=16, top=4, ff=128, groups=(4, 2), scale=2.5)),
                               tiny.attention_layer(heads=4, kv_heads=2, dim=128, vdim=64, scale=0.09, chunk=70, rot_dims=64, mlp=tiny.dense_mlp(ff=256)),
                               tiny.mlstm_layer(heads=1, dim=200, vdim=256, mlp=None), tiny.mlstm_layer(heads=2, dim=64, vdim=144, mlp=None)],
                       width=128, vocab=80, scale=4.0),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", sorted(OTHER_SHAPES))
def test_other_sizes_and_layer_orders(gpu_device, dtype, shape):
    cfg = tiny.make_config(**OTHER_SHAPES[shape])
    tensors = tiny.make_tensors(cfg, seed=21)
    lm = build_lm(cfg, tensors, dtype, pages=12)
    toks = rand_tokens(90, cfg, tensors, 6)
    want = ref.FidatarRef(cfg, tensors).forward(toks)
    with lm.context_manager():
        seq = lm.open_sequence()
        whole = lm.step_sequences([(seq, toks)])
        lm.close_sequence(seq)
        seq = lm.open_sequence()
        cuts, outs, at = [40, 2, 3, 30] + [1] * 15, [], 0
        for c in cuts:
            outs.append(lm.step_sequences([(seq, toks[at:at + c])]))
            at += c
        lm.close_sequence(seq)
    assert close(whole, want, dtype), rel_err(whole, want)
    assert close(torch.cat(outs), want, dtype), rel_err(torch.cat(outs), want)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("seed", range(16))
def test_configurations_drawn_at_random(gpu_device, seed, dtype):
    """Layer kinds, orders, feed-forwards and sizes drawn from the design's whole space: a whole prompt, portions with single
    tokens, and two requests of unequal length in one batch."""
    cfg = tiny.random_config(seed)
    tensors = tiny.make_tensors(cfg, seed=100 + seed)
    lm = build_lm(cfg, tensors, dtype, pages=16)
    model = ref.FidatarRef(cfg, tensors)
    a, b = rand_tokens(120, cfg, tensors, 7), rand_tokens(45, cfg, tensors, 8)
    want_a, want_b = model.forward(a), model.forward(b)
    with lm.context_manager():
        seq = lm.open_sequence()
        whole = lm.step_sequences([(seq, a)])
        lm.close_sequence(seq)
        sa, sb = lm.open_sequence(), lm.open_sequence()
        got_a = [lm.step_sequences([(sa, a[:70])])]
        out = lm.step_sequences([(sa, a[70:72]), (sb, b[:40])])
        got_a.append(out[:2])
        got_b = [out[2:]]
        for i in range(5):
            out = lm.step_sequences([(sa, [a[72 + i]]), (sb, [b[40 + i]])])
            got_a.append(out[:1])
            got_b.append(out[1:])
        got_a.append(lm.step_sequences([(sa, a[77:])]))
        lm.close_sequence(sa)
        lm.close_sequence(sb)
    assert close(whole, want_a, dtype), (cfg, rel_err(whole, want_a))
    assert close(torch.cat(got_a), want_a, dtype), (cfg, rel_err(torch.cat(got_a), want_a))
    assert close(torch.cat(got_b), want_b, dtype), (cfg, rel_err(torch.cat(got_b), want_b))


# ---- mechanisms alone ------------------------------------------------------------------------------------------------------
class _Step:
    """What a mixer kernel needs to know about a ragged step of sequences that hold `cached` tokens and bring `new` more."""

    def __init__(self, cached, new, slots, dev):
        self.cu = torch.tensor(np.concatenate([[0], np.cumsum(new)]), dtype=torch.int32, device=dev)
        self.pos = torch.tensor(np.concatenate([np.arange(c, c + n) for c, n in zip(cached, new)]), dtype=torch.int32, device=dev)
        self.ctx = torch.tensor([c + n for c, n in zip(cached, new)], dtype=torch.int32, device=dev)
        self.slots = torch.tensor(slots, dtype=torch.int32, device=dev)
        self.max_q, self.max_ctx = max(new), max(c + n for c, n in zip(cached, new))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [72, 37, 9, 2048, 132, 4100])
@pytest.mark.parametrize("T", [1, 37])
def test_norm_after_the_sum(gpu_device, dtype, W, T):
    """The update of a sublayer for every kind of result it leaves — a tensor, the split-K slabs of its projection, a mixture's rows —
    with the stream kept or not, a second norm behind it or not, and products of the rounded row."""
    from tgis_amd import native

    g = torch.Generator().manual_seed(W + T)
    dev, alpha, eps = gpu_device, 1.9, 1e-5
    rnd = lambda *sh: torch.randn(*sh, generator=g)
    X, w, w2, dots = rnd(T, W), 1 + 0.3 * rnd(W), 1 + 0.3 * rnd(W), rnd(21, W).to(dtype)
    tol = 2e-5 if dtype == torch.float32 else 0.012

    def check(y_dev, y):
        new = ref.rms_unit(alpha * X.double() + (y.double() if y is not None else 0), eps) * w.double() if y is not None else X.double()
        gain = w.to(dev) if y is not None else None
        xd = X.to(dev).clone()
        x_out, h, z = native.post_norm_update(xd, y_dev, alpha, gain, eps, dtype, dots=dots.to(dev))
        assert x_out.data_ptr() == xd.data_ptr() and max_err(x_out, new) <= 2e-5 and max_err(h, new) <= tol
        assert max_err(z, h.double().cpu() @ dots.double().T) <= 2e-5
        xd = X.to(dev).clone()
        x_none, h2, none = native.post_norm_update(xd, y_dev, alpha, gain, eps, dtype, w2=w2.to(dev), keep_x=False)
        assert x_none is None and none is None and torch.equal(xd.cpu(), X)
        assert max_err(h2, ref.rms_unit(new, eps) * w2.double()) <= tol

    check(None, None)
    y = rnd(T, W).to(dtype)
    check(y.to(dev), y)
    S, ld = 5, (W + 31) // 32 * 32
    slabs = rnd((T + 31) // 32, S, 32, ld)
    part = native.Partial(slabs.to(dev), S, ld, T, W, None)
    part.dtype = dtype
    check(part, slabs.sum(1).reshape(-1, ld)[:T, :W])
    for k in (1, 2, 5):
        rows, pos = rnd(40, W).to(dtype), torch.randint(0, 40, (T * k,), generator=g).to(torch.int32)
        wt = torch.rand(T * k, generator=g)
        mixed = (rows.double()[pos.long()].view(T, k, W) * wt.double().view(T, k, 1)).sum(1)
        check(native.MixtureRows(rows.to(dev), pos.to(dev), wt.to(dev), k), mixed)


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_stream_begins_with_the_scaled_embedding(gpu_device, dtype):
    from tgis_amd import native

    g = torch.Generator().manual_seed(0)
    table, ids, dots = torch.randn(50, 24, generator=g).to(dtype), torch.tensor([3, 49, 0, 7]), torch.randn(6, 24, generator=g).to(dtype)
    x, h, z = native.post_norm_update(None, None, 2.0, None, 1e-5, dtype, ids=ids.to(gpu_device), table=table.to(gpu_device), emb_scale=3.0,
                                      dots=dots.to(gpu_device))
    want = table.double()[ids] * 3.0
    assert max_err(x, want) <= 1e-6 and max_err(h, want) <= (1e-6 if dtype == torch.float32 else 0.005)
    assert max_err(z, h.double().cpu() @ dots.double().T) <= 1e-5


@pytest.mark.parametrize("dtype", [torch.float16, torch.bfloat16])
@pytest.mark.parametrize("T,R,W", [(1, 1, 8), (65, 6, 72), (100, 64, 256), (33, 70, 1000), (300, 130, 136), (16, 16, 32), (700, 32, 2048)])
def test_narrow_products(gpu_device, dtype, T, R, W):
    """fp32 sums of two-byte operands, exact products: rows, outputs and channels that fill no tile."""
    from tgis_amd import native

    g = torch.Generator().manual_seed(T + R + W)
    h, w = torch.randn(T, W + 8, generator=g).to(dtype), torch.randn(R, W, generator=g).to(dtype)
    got = native.narrow_product(h.to(gpu_device)[:, :W], w.to(gpu_device))
    want = h[:, :W].double() @ w.double().T
    assert got.shape == (T, R) and float((got.double().cpu() - want).abs().max()) <= 1e-5 * W ** 0.5 * 8


@pytest.mark.parametrize("E,top,groups,keep", [(6, 2, 3, 2), (6, 2, 1, 1), (8, 3, 8, 5), (130, 8, 10, 3), (16, 16, 4, 4), (64, 6, 8, 4), (1, 1, 1, 1), (12, 1, 4, 1), (200, 64, 100, 40)])
def test_routing_by_groups(gpu_device, E, top, groups, keep):
    """The choice from logits, and the same inside the stream's update, against the definition."""
    from tgis_amd import native

    g = torch.Generator().manual_seed(E + top)
    T, W = 45, 40
    rw, X, w = torch.randn(E, W, generator=g) * W ** -0.5 * 2, torch.randn(T, W, generator=g), torch.ones(W)
    h = ref.rms_unit(X.double(), 1e-5).float()
    r = {"experts": E, "top": top, "scale": 1.7, "groups": {"count": groups, "keep": keep}}
    ref.ROUTER_MARGINS = []
    want_i, want_w = ref.route(h.double(), rw.double(), r)
    ref.ROUTER_MARGINS = None
    s = torch.sigmoid(h.double() @ rw.double().T)
    # rows near a tie (between groups, or between neighbours in the order of the chosen) are not compared
    sure = torch.ones(T, dtype=torch.bool)
    if keep < groups:
        rank = s.view(T, groups, -1).topk(min(2, E // groups), dim=-1).values.sum(-1).sort(-1, descending=True).values
        sure &= (rank[:, keep - 1] - rank[:, keep]) > 1e-5
    srt = torch.gather(s, 1, want_i)
    if top > 1:
        sure &= (srt[:, :-1] - srt[:, 1:]).min(-1).values > 1e-6
    allowed_next = s.clone().scatter_(1, want_i, -1.0)
    if keep < groups:
        kept = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, s.view(T, groups, -1).topk(min(2, E // groups), dim=-1).values.sum(-1).topk(keep, dim=-1).indices, True)
        allowed_next = torch.where(kept.repeat_interleave(E // groups, 1), allowed_next, torch.full_like(s, -1.0))
    sure &= (srt[:, -1] - allowed_next.max(-1).values) > 1e-6
    assert int(sure.sum()) > T // 2
    logits = (h @ rw.T).to(gpu_device)
    a = native.moe_choose(logits, top, groups, keep, 1.7)
    _, _, b = native.post_norm_update(X.to(gpu_device), torch.zeros(T, W, device=gpu_device), 1.0, w.to(gpu_device), 1e-5, torch.float32, dots=rw.to(gpu_device),
                                      router=(top, groups, keep, 1.7))
    for idx, wt in (a, b):
        assert torch.equal(idx.cpu().long()[sure], want_i[sure]) and float((wt.double().cpu() - want_w)[sure].abs().max()) < 1e-5


def memory_reference(proj, cols, gates, ib, fb, cap, gain, H, dk, dv, eps, gate_act=True):
    """The matrix memory of one sequence from the rounded columns of a projection: (outputs [n, H dv], S, n, m)."""
    n = proj.shape[0]
    part = lambda c, d: proj[:, c:c + H * d].double().view(n, H, d)
    q, k, v = part(cols[0], dk) * dk ** -0.5, part(cols[1], dk), part(cols[2], dv)
    soft = lambda z: cap * torch.tanh(z / cap)
    i = soft(gates[:, :H].double() + ib.double())
    f = torch.nn.functional.logsigmoid(soft(gates[:, H:].double() + fb.double()))
    S, nn, m, rows = torch.zeros(H, dk, dv, dtype=D), torch.zeros(H, dk, dtype=D), torch.zeros(H, dtype=D), []
    for t in range(n):
        S, nn, m, o = ref.matrix_memory_step(S, nn, m, q[t], k[t], v[t], i[t], f[t])
        rows.append(o)
    out = ref.rms_unit(torch.stack(rows), eps).reshape(n, H * dv) * gain.double()
    return out * torch.sigmoid(proj[:, cols[3]:cols[3] + H * dv].double()), S, nn, m


MEMORY_SIZES = [(3, 24, 40), (1, 8, 8), (2, 33, 7), (5, 4, 20), (2, 64, 64), (2, 128, 128), (4, 80, 96), (1, 200, 256), (1, 256, 16), (2, 16, 130)]
MEMORY_CUTS = [[1, 2, 30, 1, 40, 150, 76], [2, 1, 1, 33, 1, 128, 65]]


def chunks_ok(dtype, dk, dv):
    return dtype == torch.bfloat16 and dk <= 128 and dv <= 128 and dk % 8 == 0 and dv % 8 == 0


@pytest.mark.parametrize("dtype,H,dk,dv,impl", [(t, *s, i) for t in DTYPES for s in MEMORY_SIZES for i in (0, 1, 2) if i < 2 or chunks_ok(t, *s[1:])])
def test_matrix_memory_and_its_state(gpu_device, dtype, H, dk, dv, impl):
    """Two sequences in one launch, in portions of 1, 2 and more tokens, in slots with stale contents, gates of every size; the final
    state; nothing outside the two slots is written.  impl: the launcher's choice, token by token, chunks (bfloat16, head widths that
    are multiples of 8 up to 128)."""
    from tgis_amd import native

    g = torch.Generator().manual_seed(H * dk + dv)
    dev, eps, cap = gpu_device, 1e-6, 9.0
    widths = (H * dk, H * dk, H * dv, H * dv)
    cols, at = [], 8
    for w in widths:
        cols.append(at)
        at += (w + 7) // 8 * 8 + 8
    ld = at + 16
    lens = [sum(c) for c in MEMORY_CUTS]
    projs = [torch.randn(n, ld, generator=g).to(dtype) for n in lens]
    gates = [torch.randn(n, 2 * H, generator=g) * 4 for n in lens]
    ib, fb = torch.randn(H, generator=g) * 2 - 1, torch.randn(H, generator=g) * 2 + 3
    gain = 1 + 0.3 * torch.randn(H * dv, generator=g)
    want = [memory_reference(p, cols, z, ib, fb, cap, gain, H, dk, dv, eps) for p, z in zip(projs, gates)]
    state, memory = torch.full((4, H, dk, dv), 55.0, device=dev), torch.full((4, H, dk + 1), 55.0, device=dev)
    got, done = [[], []], [0, 0]
    for step in range(7):
        new = [MEMORY_CUTS[b][step] for b in range(2)]
        st = _Step(done, new, [2, 0], dev)
        x = torch.cat([projs[b][done[b]:done[b] + new[b]] for b in range(2)]).to(dev)
        z = torch.cat([gates[b][done[b]:done[b] + new[b]] for b in range(2)]).to(dev)
        out = native.matrix_memory(x, *cols, z, ib.to(dev), fb.to(dev), cap, gain.to(dev), state, memory, st.slots, st.cu, st.pos, H, dk, dv,
                                   dk ** -0.5, eps, 1e-6, max_q_len=st.max_q, impl=impl)
        got[0].append(out[:new[0]])
        got[1].append(out[new[0]:])
        done = [a + n for a, n in zip(done, new)]
    assert done == lens
    exact = dtype == torch.float32
    for b, slot in ((0, 2), (1, 0)):
        o, S, nn, m = want[b]
        assert max_err(torch.cat(got[b]), o) <= (2e-4 if exact else 0.012), b
        stol = 1e-5 if exact or impl == 1 else 1e-4
        assert max_err(state[slot], S) <= stol and max_err(memory[slot][:, :dk], nn) <= stol
        assert float((memory[slot][:, dk].double().cpu() - m).abs().max()) <= 1e-4
    for slot in (1, 3):
        assert float(state[slot].min()) == 55.0 == float(state[slot].max()) and float(memory[slot].min()) == 55.0 == float(memory[slot].max())


@pytest.mark.parametrize("dtype,impl", [(torch.float32, 1), (torch.bfloat16, 1), (torch.bfloat16, 2)])
def test_matrix_memory_keeps_a_far_write(gpu_device, dtype, impl):
    """A value written at position 3 with a large input gate and asked for 500 tokens later, through forget gates that are all but
    open; everything else writes next to nothing.  And the maximum starts at 0: before the large gate, small input gates leave the
    denominator's floor at e^0, so that the (unnormed) read-out is tiny and the eps under the norm's root shows."""
    from tgis_amd import native

    dev, n, dk, dv, cap, eps = gpu_device, 504, 16, 24, 15.0, 1e-6
    g = torch.Generator().manual_seed(3)
    proj = (torch.randn(n, 2 * dk + 2 * dv, generator=g) * 0.2).to(dtype)
    cols = [0, dk, 2 * dk, 2 * dk + dv]
    gates = torch.zeros(n, 2)
    gates[:, 0], gates[:, 1] = -9.0, 12.0
    gates[3, 0] = 9.0
    u = torch.randn(dk, generator=g)
    proj[3, dk:2 * dk] = u.to(dtype)
    proj[503, :dk] = u.to(dtype)
    mark = torch.randn(dv, generator=g)
    proj[3, 2 * dk:2 * dk + dv] = (mark * 5).to(dtype)
    proj[:, cols[3]:] = 20.0  # open output gates
    zero, one = torch.zeros(1), torch.ones(dv)
    want, *_ = memory_reference(proj, cols, gates, zero, zero, cap, one, 1, dk, dv, eps)
    o = want[503] / want[503].norm()
    assert float((o * (mark / mark.norm()).double()).sum()) > 0.999  # the oracle reads the mark
    assert float(want[2].abs().max()) < 0.3 < float(want[3].abs().max())  # far below unit size before the large gate
    for cuts in ([504], [2, 1, 500, 1], [1, 63, 64, 375, 1]):
        state, memory, at, outs = torch.full((1, 1, dk, dv), 9.0, device=dev), torch.full((1, 1, dk + 1), 9.0, device=dev), 0, []
        for c in cuts:
            st = _Step([at], [c], [0], dev)
            outs.append(native.matrix_memory(proj[at:at + c].to(dev), *cols, gates[at:at + c].to(dev), None, None, cap, one.to(dev), state, memory,
                                             st.slots, st.cu, st.pos, 1, dk, dv, dk ** -0.5, eps, 1e-6, max_q_len=c, impl=impl))
            at += c
        got = torch.cat(outs)
        tol = 1e-4 if dtype == torch.float32 else 0.01
        assert max_err(got, want) <= tol and max_err(got[503], want[503]) <= tol and max_err(got[:3], want[:3]) <= 2 * tol, cuts
    # without an output gate at all (the gates above are open)
    st = _Step([0], [n], [0], dev)
    bare = native.matrix_memory(proj.to(dev), *cols[:3], -1, gates.to(dev), None, None, cap, one.to(dev), torch.zeros(1, 1, dk, dv, device=dev),
                                torch.zeros(1, 1, dk + 1, device=dev), st.slots, st.cu, st.pos, 1, dk, dv, dk ** -0.5, eps, 1e-6, max_q_len=n, impl=impl)
    assert max_err(bare, want) <= tol


GEOMETRIES = [(6, 3, 32, 24), (8, 2, 80, 64), (4, 4, 16, 32), (2, 1, 128, 128), (3, 1, 10, 6), (16, 1, 64, 96)]


def _write_and_attend(native, dev, dtype, q, k, v, scale, chunk, freq, amp, qg, kg, pieces, sink=None, impl=0, ws=True, eps=1e-5):
    """q [n, H, dk], k [n, G, dk], v [n, G, dv] of one sequence go through norm, rotation and cache write, then attention, in the given
    portions; pages are dealt in a scrambled order.  Returns [n, H dv]."""
    from tgis_amd.utils.layers import workspace

    n, H, dk = q.shape
    G, dv = k.shape[1], v.shape[2]
    pages = (n + 31) // 32
    kp = torch.zeros((pages + 3, G, 32 * dk), dtype=dtype, device=dev)
    vp = torch.zeros((pages + 3, G, dv * 32), dtype=dtype, device=dev)
    order = torch.randperm(pages + 2, generator=torch.Generator().manual_seed(n))[:pages].to(torch.int32)
    bt = order.view(1, -1).to(dev)
    pad = -(H * dk + G * (dk + dv)) % 8
    proj_all = torch.cat([q.reshape(n, -1), k.reshape(n, -1), v.reshape(n, -1), torch.zeros(n, pad)], 1).to(dtype)
    outs, at = [], 0
    rot = 2 * len(freq)
    for c in pieces:
        proj = proj_all[at:at + c].to(dev).contiguous()
        st = _Step([at], [c], [0], dev)
        p = torch.arange(at, at + c)
        slots = (order[(p // 32)].long() * 32 + p % 32).to(torch.int32).to(dev)
        turns = native.pair_turns(st.pos, freq.to(dev)) if rot else None
        native.norm_rope_rows_kv_write(proj, 0, H * dk, H * dk + G * dk, qg.to(dev), kg.to(dev), eps, turns, amp, slots, kp, vp, H, G, dk, dv, rot)
        outs.append(native.attn_varlen_blocks(proj[:, :H * dk], kp, vp, bt, st.ctx, st.cu, H, G, dk, dv, scale, chunk=chunk,
                                              sink=sink.to(dev) if sink is not None else None, max_q_len=c, max_ctx=at + c, impl=impl,
                                              ws=workspace(dev) if ws else None))
        at += c
    assert at == n
    return torch.cat(outs)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("geom", GEOMETRIES)
@pytest.mark.parametrize("chunk", [0, 1, 33, 64, 130])
def test_block_attention_against_plain_softmax(gpu_device, dtype, geom, chunk):
    """Norm, rotation, cache write and attention with a block mask and a 1 in the denominator, in prompt portions (one long enough for
    the transposing value writer) and single tokens over scrambled pages, against the plain form."""
    from tgis_amd import native

    H, G, dk, dv = geom
    g = torch.Generator().manual_seed(H * dk + chunk)
    n = 760
    q, k, v = torch.randn(n, H, dk, generator=g) * 2, torch.randn(n, G, dk, generator=g) * 0.3, torch.randn(n, G, dv, generator=g)
    qg, kg = 1.5 + 0.3 * torch.randn(dk, generator=g), 1.2 + 0.3 * torch.randn(dk, generator=g)
    rdims = dk // 2 * 2 if H % 2 else (dk // 4) * 2
    freq, amp = ref.yarn_frequencies(700.0, rdims, tiny.SCALING)
    r16 = lambda t: t.to(dtype).double()
    pos = torch.arange(n)
    prep = lambda t, gain: ref.turn_halves(ref.rms_unit(r16(t), 1e-5) * gain.double(), pos, freq, amp)
    want = ref.attend_in_blocks(prep(q, qg), prep(k, kg), r16(v), pos, dk ** -0.5, chunk).reshape(n, H * dv)
    tol = 4e-5 if dtype == torch.float32 else 0.03
    for impl in (0, 1):  # the launcher's choice (matrix cores for two-byte models), and the general kernel
        got = _write_and_attend(native, gpu_device, dtype, q, k, v, dk ** -0.5, chunk, freq.float(), amp, qg, kg, [530, 100, 2, 31, 33, 1, 1, 3, 40] + [1] * 19,
                                sink=torch.zeros(H), impl=impl)
        assert max_err(got, want) <= tol, impl


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("geom", [(6, 3, 32, 24), (8, 2, 80, 64)])
@pytest.mark.parametrize("chunk", [50, 64, 97])
def test_attention_finds_a_planted_key_inside_its_block_only(gpu_device, dtype, geom, chunk):
    """One key at a block's first and one at another block's last position where every query points, their values far from all
    others: a query sees one iff it lies in the same block and not before it — in a prompt, in portions that end at block and page
    borders and in single decoded tokens."""
    from tgis_amd import native

    H, G, dk, dv = geom
    g = torch.Generator().manual_seed(chunk)
    n = 8 * chunk
    first, last = 3 * chunk, 6 * chunk - 1
    u = torch.randn(G, dk, generator=g)
    q = u.repeat_interleave(H // G, 0)[None] + 0.05 * torch.randn(n, H, dk, generator=g)
    k, v = torch.randn(n, G, dk, generator=g), torch.randn(n, G, dv, generator=g)
    k[first], k[last] = u, u
    v[first], v[last] = 50.0, -50.0
    pos = torch.arange(n)
    gain, none = torch.full((dk,), (14.0 * dk ** -0.5) ** 0.5), torch.zeros(0)
    sees_first = (pos >= first) & (pos < first + chunk)
    sees_last = pos == last
    for pieces in ([n], [first, 1, chunk - 2, 1, 1, n - first - chunk - 1], [last, 1, 1, 1, n - last - 3], [first + 1] + [1] * (chunk + 2) + [n - first - chunk - 3]):
        got = _write_and_attend(native, gpu_device, dtype, q, k, v, 1.0, chunk, none, 1.0, gain, gain, pieces, sink=torch.zeros(H)).float().cpu().view(n, H, dv)
        share = got.mean(-1) / 50.0
        assert float(share[sees_first].min()) > 0.85, pieces[:3]
        assert float(share[sees_last].max()) < -0.85, pieces[:3]
        assert float(share[~sees_first & ~sees_last].abs().max()) < 0.1, pieces[:3]


def test_the_one_in_the_denominator(gpu_device):
    """Keys that score zero: with three visible keys the values' weights sum to 3 / 4; without a sink to one; at a block's first
    position to 1 / 2."""
    from tgis_amd import native

    n, v = 40, torch.ones(40, 1, 32)
    one = torch.ones(16)
    for dtype in DTYPES:
        for impl in (0, 1):
            args = (native, gpu_device, dtype, torch.zeros(n, 2, 16), torch.randn(n, 1, 16), v, 1.0, 3, torch.zeros(0), 1.0, one, one, [35, 1, 2, 2])
            got = _write_and_attend(*args, sink=torch.zeros(2), impl=impl).float().cpu().view(n, 2, 32)
            want = torch.tensor([[1 / 2, 2 / 3, 3 / 4][i % 3] for i in range(n)]).view(n, 1, 1).expand(n, 2, 32)
            assert torch.allclose(got, want, atol=3e-3)
            assert torch.allclose(_write_and_attend(*args, impl=impl).float().cpu(), torch.ones(n, 64), atol=3e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("N,K", [(88, 72), (33, 37), (512, 256), (130, 1024)])
@pytest.mark.parametrize("T", [1, 37, 200, 300])
def test_squared_relu_feed_forward(gpu_device, dtype, N, K, T):
    from tgis_amd import native
    from tgis_amd.utils.layers import workspace
    from tgis_amd.utils.mixers import ActivatedMLP
    from tgis_amd.utils.weights import DictWeights

    g = torch.Generator().manual_seed(N + T)
    t = {"f.up": (torch.randn(N, K, generator=g) * K ** -0.5).to(dtype), "f.down": (torch.randn(K, N, generator=g) * N ** -0.5).to(dtype)}
    h = torch.randn(T, K, generator=g).to(dtype)
    mlp = ActivatedMLP(DictWeights(t, device=gpu_device, dtype=dtype, process_group=_One()), "f", act="relu2")
    want = ref.unit(h.double(), {n[2:]: v.double() for n, v in t.items()})
    assert max_err(mlp(h.to(gpu_device)), want) <= (2e-5 if dtype == torch.float32 else 0.02)
    z = torch.randn(T, N, generator=g).to(dtype).to(gpu_device)
    assert torch.equal(native.relu2(z), (z.float().clamp(min=0) ** 2).to(dtype))
    if mlp.up.streams and T <= 256:  # the epilogue form has the bits of the two steps
        hd = h.to(gpu_device)
        assert torch.equal(native.dense_gemm_relu2(hd, mlp.up.prepared, workspace(gpu_device)), native.relu2(native.dense_gemm(hd, mlp.up.prepared, workspace(gpu_device))))


class _One:
    def size(self):
        return 1

    def rank(self):
        return 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [5, 37, 600])
@pytest.mark.parametrize("E,k,W,ff,groups,keep", [(6, 2, 72, 40, 3, 2), (12, 4, 64, 96, 4, 2), (3, 3, 37, 21, 1, 1), (1, 1, 40, 16, 1, 1), (4, 2, 96, 160, 4, 3)])
def test_mixture_of_squared_relu_units(gpu_device, dtype, T, E, k, W, ff, groups, keep):
    """Routed plain units, summed by the combine launch and left to the stream's update."""
    from tgis_amd import native
    from tgis_amd.utils.mixers import RoutedExperts
    from tgis_amd.utils.weights import DictWeights

    f = tiny.moe_mlp(experts=E, top=k, ff=ff, groups=(groups, keep), scale=1.3)
    tensors = tiny.make_tensors(tiny.make_config([tiny.mlstm_layer(mlp=f)], width=W), seed=E)
    p = {n[len("l0.mlp."):]: v.double() for n, v in tensors.items() if n.startswith("l0.mlp.")}
    g = torch.Generator().manual_seed(T)
    h = torch.randn(T, W, generator=g).to(dtype)
    s = torch.sigmoid(h.double() @ p["router"].T)
    sure = torch.ones(T, dtype=torch.bool)  # rows near a tie are not compared
    rank = s.view(T, groups, -1).topk(min(2, E // groups), dim=-1).values.sum(-1)
    if keep < groups:
        r = rank.sort(-1, descending=True).values
        sure &= (r[:, keep - 1] - r[:, keep]) > 1e-3
        ok = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, rank.topk(keep, dim=-1).indices, True).repeat_interleave(E // groups, 1)
        s = torch.where(ok, s, torch.zeros_like(s))
    if k < E:
        b = s.sort(-1, descending=True).values
        sure &= (b[:, k - 1] - b[:, k]) > 1e-3
    want = ref.mixture(h.double(), p, f)
    w = DictWeights(tensors, device=gpu_device, dtype=dtype, process_group=_One())
    ex = RoutedExperts(w, "l0.mlp", experts=E, top=k, shared=False, weight_on_input=False, unit="relu2", groups=groups, keep_groups=keep, grouped_sigmoid=1.3)
    got = ex(h.to(gpu_device)).double().cpu()
    tol = 2e-5 if dtype == torch.float32 else 0.03
    assert float((got - want)[sure].abs().max()) <= tol * float(want.abs().max())
    rows = ex(h.to(gpu_device), defer=True)
    X = torch.randn(T, W, generator=g)
    x, _, _ = native.post_norm_update(X.to(gpu_device), rows, 2.0, torch.ones(W, device=gpu_device), 1e-5, dtype)
    assert max_err(x[sure.to(gpu_device)], ref.rms_unit(2.0 * X.double() + want, 1e-5)[sure]) <= tol


@pytest.mark.parametrize("dtype", [torch.float16, torch.bfloat16])
@pytest.mark.parametrize("tile", [32, 128])
def test_grouped_products_with_squared_relu(gpu_device, dtype, tile):
    from tgis_amd import native

    g = torch.Generator().manual_seed(tile)
    dev, T, k, E, N, K = gpu_device, 450, 2, 5, 200, 96
    idx = torch.stack([torch.randperm(E, generator=g)[:k] for _ in range(T)]).to(torch.int32)
    h, w = torch.randn(T, K, generator=g).to(dtype), (torch.randn(E, N, K, generator=g) * K ** -0.5).to(dtype)
    want = torch.stack([ref.relu2(h[i // k].double() @ w[int(e)].double().T) for i, e in enumerate(idx.view(-1))])
    srt, te, pos, nt = native.moe_align(idx.to(dev), E, tile)
    out = native.moe_gemm(h.to(dev), native.MoeWeight(w.to(dev), glu=False), te, nt, srt.shape[0], sorted_=srt, pair_div=k, tile_rows=tile, relu2=True)
    assert max_err(out[pos.long()], want) <= (0.01 if dtype == torch.bfloat16 else 0.003)


# ---- generation through the serving entry points ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk", [0, 16])
def test_greedy_generation_through_batches(gpu_device, std, dtype, chunk, monkeypatch):
    """from_pb -> generate_token(first) -> decode steps (captured graphs) with a second batch prefilled, concatenated and
    one request pruned on the way; prompts prefilled whole or in portions of 16.  Token ids against a teacher-forced greedy
    continuation."""
    from tgis_amd.testing import SyntheticTokenizer, make_batch_pb

    cfg, tensors = std
    monkeypatch.setenv("TGIS_PREFILL_CHUNK", str(chunk))
    tok = SyntheticTokenizer(cfg["vocab"])
    lm = build_lm(cfg, tensors, dtype, pages=40, slots=6, tokenizer=tok)
    steps = 12
    with lm.context_manager():
        b1, errs = lm.batch_type.from_pb(make_batch_pb([37, 5, 50], steps, batch_id=0), tok, lm.dtype, lm.device, None, None, True)
        assert not errs
        prompts = {r.id: b1.all_input_ids_tensor[i, :l].tolist() for i, (r, l) in enumerate(zip(b1.requests, b1.input_lengths))}
        out = {r.id: [] for r in b1.requests}
        for t in lm.generate_token(b1, first=True)[0]:
            out[t.request_id].append(t.token_id)
        for _ in range(3):
            for t in lm.generate_token(b1)[0]:
                out[t.request_id].append(t.token_id)
        b2, _ = lm.batch_type.from_pb(make_batch_pb([20, 33], steps, batch_id=1, first_request_id=3), tok, lm.dtype, lm.device, None, None, True)
        for i, (r, l) in enumerate(zip(b2.requests, b2.input_lengths)):
            prompts[r.id] = b2.all_input_ids_tensor[i, :l].tolist()
            out[r.id] = []
        for t in lm.generate_token(b2, first=True)[0]:
            out[t.request_id].append(t.token_id)
        batch = lm.batch_type.concatenate([b1, b2])
        for _ in range(3):
            for t in lm.generate_token(batch)[0]:
                out[t.request_id].append(t.token_id)
        batch = lm.batch_type.prune(batch, [1])
        assert lm.state_cache.free_slots == 6 - 4
        for _ in range(4):
            for t in lm.generate_token(batch)[0]:
                out[t.request_id].append(t.token_id)
        batch.release()
    assert lm.kv_cache.free_pages == 40 and lm.state_cache.free_slots == 6
    # float32: the oracle, fed the engine's own tokens — at every step the engine's choice must be the oracle's argmax.
    # bfloat16: the prompts here are not drawn to keep routers away from ties, so the yardstick is the same checkpoint stepped
    # sequence by sequence through step_sequences in bfloat16 (no batches, no captured graphs, no pruning); a choice may differ
    # only within the bf16 bound on a row.
    model = ref.FidatarRef(cfg, tensors)
    plain = build_lm(cfg, tensors, dtype, pages=40, slots=2) if dtype == torch.bfloat16 else None
    for rid, ids in out.items():
        if plain is None:
            st = model.new_state()
            step = lambda toks: model.advance(st, toks)[-1]
        else:
            seq = plain.open_sequence()
            step = lambda toks: plain.step_sequences([(seq, toks)])[-1].double().cpu()
        with (plain.context_manager() if plain is not None else torch.no_grad()):
            logits = step(prompts[rid])
            for k, t in enumerate(ids):
                best = int(logits.argmax())
                if t != best:
                    gap = float(logits[best] - logits[t])
                    assert dtype == torch.bfloat16 and gap < TOL[dtype] * float(logits.std()), (rid, k, t, best, gap)
                logits = step([t])
        if plain is not None:
            plain.close_sequence(seq)


# ---- the trace runner, as a user starts it ---------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_runner_replays_a_schedule(gpu_device, tmp_path, dtype):
    """A checkpoint folder of its own shape written to disk and replayed by bin/trace_run in a child process: requests admitted
    at different steps, portions beside single tokens, a request that sits a step out, a pool of 6 pages for 3 live requests,
    slots and pages handed on to later requests."""
    from safetensors.torch import save_file

    layers = [tiny.attention_layer(heads=8, kv_heads=4, dim=16, vdim=32, scale=0.25, chunk=20, rot_dims=4, mlp=tiny.moe_mlp(experts=4, top=2, ff=32, groups=(2, 1))),
              tiny.mlstm_layer(heads=2, dim=16, vdim=32, mlp=tiny.moe_mlp(experts=5, top=3, ff=24, groups=None)),
              tiny.mlstm_layer(heads=4, dim=8, vdim=8, mlp=tiny.dense_mlp(ff=48))]
    cfg = tiny.make_config(layers, width=64, vocab=70, eps=1e-6)
    tensors = tiny.make_tensors(cfg, seed=11)
    model_dir = tmp_path / "model"
    model_dir.mkdir()
    (model_dir / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in tensors.items()}, str(model_dir / "model.safetensors"))
    prompts = {"a": rand_tokens(60, cfg, tensors, 1), "b": rand_tokens(33, cfg, tensors, 2), "c": rand_tokens(64, cfg, tensors, 3), "d": rand_tokens(40, cfg, tensors, 4)}
    model = ref.FidatarRef(cfg, tensors)
    want = {k: model.forward(v) for k, v in prompts.items()}
    schedule = [[("a", 31)], [("a", 2), ("b", 30)], [("a", 1), ("b", 1), ("c", 33)], [("a", 26), ("c", 1)], [("b", 2), ("c", 30)],
                [("d", 2)], [("d", 37), ("c", 0)], [("d", 1)]]
    done = {k: 0 for k in prompts}
    lines, expect = [], []
    for n, step in enumerate(schedule):
        entries, rows, end = [], [], []
        for rid, cnt in step:
            if cnt == 0:
                continue
            lo = done[rid]
            entries.append({"id": rid, "tokens": prompts[rid][lo:lo + cnt], "want": list(range(cnt))})
            rows.append(want[rid][lo:lo + cnt])
            done[rid] += cnt
            if done[rid] == len(prompts[rid]):
                end.append(rid)
        lines.append(json.dumps({"step": n, "entries": entries, "end": end}))
        expect.append(torch.cat(rows))
    out_dir = tmp_path / "out"
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(model_dir), "--dtype", dtype,
                        "--out", str(out_dir), "--max-tokens", "192", "--slots", "3"],
                       input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=280)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done ")] == [f"done {n}" for n in range(len(schedule))]
    dt = torch.float32 if dtype == "float32" else torch.bfloat16
    for n, e in enumerate(expect):
        got = torch.from_numpy(np.fromfile(out_dir / f"{n}.f32", dtype="<f4").reshape(e.shape).copy())
        assert close(got, e, dt), n
