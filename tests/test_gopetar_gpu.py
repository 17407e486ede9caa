"""GPU: the Gopetar family on the kernels (FlashCausalLM + utils/mixers.py + csrc/hyper_streams, min_gru, head_product, attn_varlen,
moe) against the plain float64 restatement in oracle/gopetar_ref.py, on small seeded checkpoints of their own sizes.

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

from oracle import gopetar_ref as ref
from oracle import gopetar_tiny as tiny

pytestmark = pytest.mark.gpu

TOL = {torch.float32: 2e-4, torch.bfloat16: 0.15}
DTYPES = [torch.float32, torch.bfloat16]
D = torch.float64


def build_lm(cfg, tensors, dtype, pages=64, slots=4, tokenizer=None):
    from tgis_amd.inference_engine.synthetic import InferenceEngine
    from tgis_amd.models.custom_modeling.flash_gopetar_modeling import GopetarConfig
    from tgis_amd.models.flash_causal_lm import FlashCausalLM

    eng = InferenceEngine({k: v.clone() for k, v in tensors.items()}, GopetarConfig(**cfg), dtype, None, tokenizer=tokenizer)
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
@pytest.mark.parametrize("n", [75, 300, 700])
def test_whole_prompt_matches_oracle_layer_by_layer(gpu_device, std, dtype, n):
    """75 tokens: the decode-sized GEMM path; 300: the library GEMMs; 700: the transposing value writers.  All are longer than every
    window of the configuration."""
    cfg, tensors = std
    lm = build_lm(cfg, tensors, dtype)
    toks = rand_tokens(n, cfg, tensors, 1)
    want_trace = []
    want = ref.GopetarRef(cfg, tensors).forward(toks, want_trace)
    with lm.context_manager():
        seq, trace = lm.open_sequence(), []
        got = lm.step_sequences([(seq, toks)], residual_trace=trace)
        lm.close_sequence(seq)
    assert len(trace) == len(want_trace) == 5
    for r, (g, w) in enumerate(zip(trace, want_trace)):
        scale = float(w.abs().max())
        assert float((g.double().cpu() - w).abs().max()) <= (1e-4 if dtype == torch.float32 else 0.08) * scale, r
    assert close(got, want, dtype), rel_err(got, want)


@pytest.mark.parametrize("dtype", DTYPES)
def test_token_by_token_and_portions_equal_whole(gpu_device, std, dtype):
    cfg, tensors = std
    lm = build_lm(cfg, tensors, dtype)
    toks = rand_tokens(150, cfg, tensors, 2)
    want = ref.GopetarRef(cfg, tensors).forward(toks)
    for cuts in ([1] * 150, [2] * 75, [3, 2, 31, 33, 1, 2, 64, 5, 9], [97, 2, 2, 2, 47], [149, 1]):
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
    model = ref.GopetarRef(cfg, tensors)
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
    want = ref.GopetarRef(cfg, tensors).forward(toks)
    with lm.context_manager():
        seq = lm.open_sequence()
        got = torch.cat([lm.step_sequences([(seq, toks[:2])]), lm.step_sequences([(seq, toks[2:])])])
        lm.close_sequence(seq)
    assert close(got, want, torch.float32), rel_err(got, want)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(gpu_device, std, dtype):
    """220 single-token steps behind a short prompt: windows pass over decoded tokens, states are carried all the way."""
    cfg, tensors = std
    lm = build_lm(cfg, tensors, dtype)
    toks = rand_tokens(240, cfg, tensors, 5)
    want = ref.GopetarRef(cfg, tensors).forward(toks)
    with lm.context_manager():
        seq = lm.open_sequence()
        outs = [lm.step_sequences([(seq, toks[:20])])] + [lm.step_sequences([(seq, [t])]) for t in toks[20:]]
        lm.close_sequence(seq)
    assert close(torch.cat(outs), want, dtype), rel_err(torch.cat(outs), want)


# sizes that the standard configuration happens to make equal, one, or a multiple of eight; other layer orders
OTHER_SHAPES = {
    "one_stream": dict(layers=[tiny.latent_layer(heads=1, dim=8, vdim=8, kv_rank=16, q_rank=16, mlp=None), tiny.pair_layer(mlp=tiny.moe_mlp(experts=1, top=1))],
                       width=40, vocab=50, streams=1, scale=1.0),
    "two_streams_only_pairs": dict(layers=[tiny.pair_layer(left=tiny.attention_part(heads=2, kv_heads=1, dim=12, vdim=20, window=1, rot_dims=4), width=33),
                                           tiny.pair_layer(left=tiny.attention_part(heads=8, kv_heads=4, dim=24, vdim=8, window=33, rot_dims=0), width=8,
                                                           mlp=tiny.moe_mlp(experts=9, top=4, ff=24, shared_ff=20))],
                                   width=24, vocab=33, streams=2, scale=16.0),
    "four_streams_only_latents": dict(layers=[tiny.latent_layer(heads=5, dim=12, vdim=20, kv_rank=20, q_rank=12, mlp=tiny.moe_mlp(experts=2, top=2, ff=16)),
                                              tiny.latent_layer(heads=2, dim=20, vdim=12, kv_rank=20, q_rank=8, kv_from=0, mlp=tiny.moe_mlp(experts=3, top=1, ff=20, shared_ff=None)),
                                              tiny.latent_layer(heads=7, dim=8, vdim=8, kv_rank=20, q_rank=9, kv_from=0, mlp=None)],
                                      width=36, vocab=41, streams=4, scale=0.5),
    "seven_streams_odd_width": dict(layers=[tiny.pair_layer(left=tiny.attention_part(heads=3, kv_heads=3, dim=10, vdim=6, window=64, rot_dims=6), width=21,
                                                            mlp=tiny.moe_mlp(experts=3, top=2, ff=21, shared_ff=11)),
                                            tiny.latent_layer(heads=2, dim=6, vdim=10, kv_rank=11, q_rank=7, mlp=tiny.moe_mlp(experts=4, top=3, ff=10, shared_ff=13))],
                                    width=37, vocab=41, streams=7, scale=3.0),
    "wide_heads": dict(layers=[tiny.pair_layer(left=tiny.attention_part(heads=4, kv_heads=2, dim=128, vdim=64, scale=0.08, window=70, rot_dims=64), width=256,
                                               mlp=tiny.moe_mlp(experts=16, top=4, ff=128, shared_ff=128)),
                               tiny.latent_layer(heads=8, dim=64, vdim=128, kv_rank=256, q_rank=192, scale=0.12, mlp=None),
                               tiny.latent_layer(heads=16, dim=32, vdim=32, kv_rank=256, q_rank=64, scale=0.2, kv_from=1, mlp=tiny.moe_mlp(ff=64, shared_ff=64))],
                       width=128, vocab=80, streams=3, scale=4.0),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", sorted(OTHER_SHAPES))
def test_other_sizes_and_layer_orders(gpu_device, dtype, shape):
    cfg = tiny.make_config(**OTHER_SHAPES[shape])
    tensors = tiny.make_tensors(cfg, seed=21)
    lm = build_lm(cfg, tensors, dtype, pages=12)
    toks = rand_tokens(90, cfg, tensors, 6)
    want = ref.GopetarRef(cfg, tensors).forward(toks)
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
    """Layer kinds, orders, stream counts and sizes drawn from the design's whole space: a whole prompt, portions with single
    tokens, and two requests of unequal length in one batch."""
    cfg = tiny.random_config(seed)
    tensors = tiny.make_tensors(cfg, seed=100 + seed)
    lm = build_lm(cfg, tensors, dtype, pages=16)
    model = ref.GopetarRef(cfg, tensors)
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
@pytest.mark.parametrize("streams,W", [(1, 72), (2, 64), (3, 37), (4, 2048), (5, 20), (8, 132), (3, 9)])
@pytest.mark.parametrize("T", [1, 37])
def test_stream_mix_and_norm(gpu_device, dtype, streams, W, T):
    """The update of a sublayer and the normed input of the next one in one launch, for every kind of result a sublayer leaves:
    a tensor, the split-K slabs of its projection, a mixture's rows with a gated shared row (a tensor or slabs), and none."""
    from tgis_amd import native

    g = torch.Generator().manual_seed(streams * W + T)
    dev, s = gpu_device, streams
    rnd = lambda *sh: torch.randn(*sh, generator=g)
    X = rnd(T, s, W)
    c = {"mix": rnd(s, s), "out": rnd(s), "in": rnd(s), "gain": torch.tensor([0.8])}
    cur, nxt = torch.cat([c["mix"].reshape(-1), c["out"]]).to(dev), torch.cat([c["in"], c["gain"]]).to(dev)
    tol = 2e-5 if dtype == torch.float32 else 0.012

    def check(y_dev, y):
        if y is None:
            new = X.double()
        else:
            new = torch.einsum("ab,taw->tbw", c["mix"].double(), X.double()) + c["out"].double()[None, :, None] * y.double()[:, None]
        u = torch.einsum("a,taw->tw", c["in"].double(), new)
        want = ref.rms_unit(u, 1e-5) * 0.8
        xd = X.to(dev).clone()
        x_out, h = native.hyper_update(xd, y_dev, cur if y is not None else None, nxt, 1e-5, dtype)
        assert x_out.data_ptr() == xd.data_ptr()
        assert float((x_out.double().cpu() - new).abs().max()) <= 2e-5 * float(new.abs().max())
        assert float((h.double().cpu() - want).abs().max()) <= tol * float(want.abs().max())

    check(None, None)
    y = rnd(T, W).to(dtype)
    check(y.to(dev), y)
    S, ld = 5, (W + 31) // 32 * 32
    slabs = rnd((T + 31) // 32, S, 32, ld)
    part = native.Partial(slabs.to(dev), S, ld, T, W, None)
    part.dtype = dtype
    y_sl = slabs.sum(1).reshape(-1, ld)[:T, :W]
    check(part, y_sl)
    for k in (1, 2, 5):
        rows, pos = rnd(40, W).to(dtype), torch.randint(0, 40, (T * k,), generator=g).to(torch.int32)
        w, gate, sh = torch.rand(T * k, generator=g), torch.rand(T, generator=g), rnd(T, W).to(dtype)
        mixed = (rows.double()[pos.long()].view(T, k, W) * w.double().view(T, k, 1)).sum(1)
        check(native.MixtureRows(rows.to(dev), pos.to(dev), w.to(dev), k), mixed)
        check(native.MixtureRows(rows.to(dev), pos.to(dev), w.to(dev), k, sh.to(dev), gate.to(dev)), mixed + gate.double()[:, None] * sh.double())
        check(native.MixtureRows(rows.to(dev), pos.to(dev), w.to(dev), k, part, gate.to(dev)), mixed + gate.double()[:, None] * y_sl.double())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,E,k,softmax_top,gate", [(72, 6, 2, True, True), (37, 3, 3, True, False), (256, 130, 8, False, True), (64, 1, 1, True, True)])
def test_routing_inside_the_stream_update(gpu_device, dtype, W, E, k, softmax_top, gate):
    """The update's own routing against the router launch on the same row, and against its definition."""
    from tgis_amd import native

    g = torch.Generator().manual_seed(W + E)
    dev, T, s = gpu_device, 33, 2
    X, y = torch.randn(T, s, W, generator=g), torch.randn(T, W, generator=g).to(dtype)
    cur, nxt = torch.randn(s * s + s, generator=g), torch.cat([torch.randn(s, generator=g), torch.tensor([1.1])])
    rw, sg = torch.randn(E, W, generator=g) * W ** -0.5, torch.randn(W, generator=g) * W ** -0.5
    sg = sg if gate else None
    new = torch.einsum("ab,taw->tbw", cur[:s * s].view(s, s).double(), X.double()) + cur[s * s:].double()[None, :, None] * y.double()[:, None]
    h = ref.rms_unit(torch.einsum("a,taw->tw", nxt[:s].double(), new), 1e-5) * nxt[s].double()
    logits = h @ rw.double().T
    _, _, (idx, wt, gt) = native.hyper_update(X.to(dev), y.to(dev), cur.to(dev), nxt.to(dev), 1e-5, dtype,
                                              router=(rw.to(dev), sg.to(dev) if gate else None, k, softmax_top))
    ri, rwt, rg = native.moe_route(h.float().to(dev), rw.to(dev), sg.to(dev) if gate else None, k, softmax_top=softmax_top)
    val, want = logits.topk(k, dim=-1)
    ww = torch.softmax(val, -1) if softmax_top else torch.sigmoid(val)
    for i, w in ((idx, wt), (ri, rwt)):
        sure = torch.ones(T, dtype=torch.bool)
        if k < E:
            b = logits.sort(-1, descending=True).values[:, :k + 1]
            sure = (b[:, :-1] - b[:, 1:]).min(-1).values > 1e-4
        assert torch.equal(i.cpu().long()[sure], want[sure]) and float((w.double().cpu() - ww)[sure].abs().max()) < 1e-4
    if gate:
        for x in (gt, rg):
            assert float((x.double().cpu() - torch.sigmoid(h @ sg.double())).abs().max()) < 1e-5
    else:
        assert gt is None


@pytest.mark.parametrize("dtype", DTYPES)
def test_streams_begin_as_copies_of_the_embedding(gpu_device, dtype):
    from tgis_amd import native

    g = torch.Generator().manual_seed(0)
    table, ids = torch.randn(50, 24, generator=g).to(dtype), torch.tensor([3, 49, 0, 7])
    nxt = torch.tensor([0.5, -2.0, 0.25, 1.5])
    X, h = native.hyper_update(None, None, None, nxt.to(gpu_device), 1e-5, dtype, ids=ids.to(gpu_device), table=table.to(gpu_device), emb_scale=3.0, streams=3)
    x = table.double()[ids] * 3.0
    assert torch.allclose(X.double().cpu(), x[:, None].repeat(1, 3, 1), atol=1e-5)
    want = ref.rms_unit(x * -1.25, 1e-5) * 1.5
    assert float((h.double().cpu() - want).abs().max()) <= (1e-5 if dtype == torch.float32 else 0.02) * float(want.abs().max())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [88, 33, 256, 8])
def test_min_gru_and_its_state(gpu_device, dtype, width):
    """Two sequences in one launch, in portions of 1, 2 and more tokens up to several rounds of the kernel, in slots with stale
    contents; the final state; nothing outside the two slots is written."""
    from tgis_amd import native

    g = torch.Generator().manual_seed(width)
    dev, lens, W = gpu_device, [700, 431], width
    cols = [4, 4 + W + 2, 4 + 2 * W + 10]
    ld = cols[2] + W + 6
    projs = [(torch.randn(n, ld, generator=g) * 1.5 - 0.3).to(dtype) for n in lens]
    want, S_end = [], []
    for p in projs:
        part = lambda c: p[:, c:c + W].double()
        zz, u = torch.sigmoid(part(cols[0])), part(cols[1])
        S, rows = torch.zeros(W, dtype=D), []
        for t in range(p.shape[0]):
            cand = torch.where(u[t] >= 0, u[t] + 0.5, torch.sigmoid(u[t]))
            S = (1 - zz[t]) * S + zz[t] * cand
            rows.append(S)
        want.append(torch.stack(rows) * ref.silu(part(cols[2])) * 0.7)
        S_end.append(S)
    state = torch.full((4, W), 55.0, device=dev)
    cuts = [[1, 2, 30, 1, 40, 300, 326], [2, 1, 1, 33, 1, 128, 265]]
    got, at = [[], []], [0, 0]
    for step in range(7):
        new = [cuts[b][step] for b in range(2)]
        st = _Step(at, new, [2, 0], dev)
        x = torch.cat([projs[b][at[b]:at[b] + new[b]] for b in range(2)]).to(dev)
        out = native.min_gru_scan(x, cols[0], cols[1], cols[2], state, st.slots, st.cu, st.pos, W, out_scale=0.7, max_q_len=st.max_q)
        got[0].append(out[:new[0]])
        got[1].append(out[new[0]:])
        at = [a + n for a, n in zip(at, new)]
    assert at == lens
    tol = 1e-5 if dtype == torch.float32 else 0.01
    for b, slot in ((0, 2), (1, 0)):
        assert float((torch.cat(got[b]).double().cpu() - want[b]).abs().max()) <= tol * float(want[b].abs().max())
        assert float((state[slot].double().cpu() - S_end[b]).abs().max()) <= 1e-5 * float(S_end[b].abs().max())
    assert float(state[1].min()) == 55.0 == float(state[3].max())


def test_min_gru_keeps_a_far_write(gpu_device):
    """A value written wholly at the first position and kept through 900 tokens whose gates are all but closed."""
    from tgis_amd import native

    dev, n, W = gpu_device, 901, 16
    z = torch.full((n, W), -9.0)
    z[0, 5], x, gate = 12.0, torch.zeros(n, W), torch.zeros(n, W)
    x[0, 5], gate[n - 1] = 40.0, 30.0
    proj = torch.cat([z, x, gate], 1).to(dev)
    keep = float((1 - torch.sigmoid(torch.tensor(-9.0, dtype=D))) ** 900)
    fresh = 0.5 * (1 - keep)  # what the closed gates let in of the candidate 1/2
    for cuts in ([901], [1, 899, 1], [300, 2, 599]):
        state, at, outs = torch.zeros(1, W, device=dev), 0, []
        for c in cuts:
            st = _Step([at], [c], [0], dev)
            outs.append(native.min_gru_scan(proj[at:at + c], 0, W, 2 * W, state, st.slots, st.cu, st.pos, W, max_q_len=c))
            at += c
        o = torch.cat(outs)[n - 1] / 30.0
        assert abs(float(o[5]) / (40.5 * keep + fresh) - 1) < 1e-4 and abs(float(o[4]) / fresh - 1) < 2e-3


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,N,K", [(3, 40, 24), (5, 11, 6), (8, 256, 64), (16, 32, 256), (1, 8, 8), (2, 100, 20)])
@pytest.mark.parametrize("T", [1, 33, 200])
def test_head_product(gpu_device, dtype, H, N, K, T):
    """One matrix per head, heads at strides of their own on both sides; what lies between them is not touched."""
    from tgis_amd import native

    g = torch.Generator().manual_seed(H * N + T)
    hx, ho = K + 3 * (K % 8 != 0) + 8, N + 5
    x, w = torch.randn(T, H * hx, generator=g).to(dtype), (torch.randn(H, N, K, generator=g) * K ** -0.5).to(dtype)
    out = torch.full((T, H * ho), 7.0, dtype=dtype, device=gpu_device)
    native.head_product(x.to(gpu_device), hx, w.to(gpu_device), out, ho)
    want = torch.einsum("thk,hnk->thn", x.view(T, H, hx)[:, :, :K].double(), w.double())
    got = out.view(T, H, ho)
    tol = 1e-5 if dtype == torch.float32 else 0.01
    assert float((got[:, :, :N].double().cpu() - want).abs().max()) <= tol * float(want.abs().max())
    assert float(got[:, :, N:].float().min()) == 7.0 == float(got[:, :, N:].float().max())


GEOMETRIES = [(6, 3, 32, 24), (8, 2, 80, 64), (4, 4, 16, 32), (2, 1, 128, 128), (3, 1, 10, 6), (16, 1, 64, 96)]


def _write_and_attend(native, dev, dtype, q, k, v, scale, window, freq, vfreq, pieces, sink=None, softcap=0.0, impl=0, ws=True, out_scale=1.0):
    """q [n, H, dk], k [n, G, dk], v [n, G, dv] of one sequence go through rotation and cache write, then attention, in the given
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
    for c in pieces:
        proj = proj_all[at:at + c].to(dev).contiguous()
        st = _Step([at], [c], [0], dev)
        p = torch.arange(at, at + c)
        slots = (order[(p // 32)].long() * 32 + p % 32).to(torch.int32).to(dev)
        kc, vc = H * dk, H * dk + G * dk
        turns = None
        fr = freq.to(dev) if freq is not None else None
        rot = 2 * len(freq) if freq is not None else 0
        if vfreq is not None:
            turns = native.pair_turns(st.pos, vfreq.to(dev))
            native.rope_rows_turned_kv_write(proj, 0, kc, vc, fr, st.pos, slots, kp, vp, H, G, dk, dv, rot, turns)
        else:
            native.rope_rows_kv_write(proj, 0, kc, vc, fr, st.pos, slots, kp, vp, H, G, dk, dv, rot)
        outs.append(native.attn_varlen_turned(proj[:, :H * dk], kp, vp, bt, st.ctx, st.cu, H, G, dk, dv, scale, window=window,
                                              sink=sink.to(dev) if sink is not None else None, softcap=softcap, turns=turns, out_scale=out_scale,
                                              max_q_len=c, max_ctx=at + c, impl=impl, ws=workspace(dev) if ws else None))
        at += c
    assert at == n
    return torch.cat(outs)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("geom", GEOMETRIES)
@pytest.mark.parametrize("window,softcap", [(0, 0.0), (1, 3.0), (33, 20.0), (70, 2.0), (200, 6.0), (0, 6.0)])
def test_turned_value_attention_against_plain_softmax(gpu_device, dtype, geom, window, softcap):
    """Rotation, turned values, cache write and attention with capped scores, a sink and a window, in prompt portions (one long
    enough for the transposing value writer) and single tokens over scrambled pages, against the plain form."""
    from tgis_amd import native

    H, G, dk, dv = geom
    g = torch.Generator().manual_seed(H * dk + window)
    n = 760
    q, k, v = torch.randn(n, H, dk, generator=g) * 2, torch.randn(n, G, dk, generator=g), torch.randn(n, G, dv, generator=g)
    rdims = dk // 2 * 2 if H % 2 else (dk // 4) * 2
    freq, vfreq = ref.pair_frequencies(700.0, rdims, tiny.SCALING), ref.pair_frequencies(700.0, dv)
    sink = torch.randn(H, generator=g) + 1.0
    r16 = lambda t: t.to(dtype).double()
    pos = torch.arange(n)
    o = ref.attend(ref.turn_pairs(r16(q), pos, freq), ref.turn_pairs(r16(k), pos, freq), ref.turn_pairs(r16(v), pos, vfreq), pos, dk ** -0.5, window, softcap, sink.double())
    want = ref.turn_pairs(o, pos, vfreq, -1.0).reshape(n, H * dv) * 0.7
    tol = 4e-5 if dtype == torch.float32 else 0.03
    for impl in (0, 1):  # the launcher's choice (matrix cores for two-byte models), and the general kernel
        got = _write_and_attend(native, gpu_device, dtype, q, k, v, dk ** -0.5, window, freq.float(), vfreq.float(), [530, 100, 2, 31, 33, 1, 1, 3, 40] + [1] * 19,
                                sink=sink, softcap=softcap, impl=impl, out_scale=0.7)
        assert float((got.double().cpu() - want).abs().max()) <= tol * float(want.abs().max()), impl


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("geom", [(6, 3, 32, 24), (8, 2, 80, 64)])
@pytest.mark.parametrize("window", [40, 64, 97])
def test_attention_finds_a_planted_key_inside_its_window_only(gpu_device, dtype, geom, window):
    """One key among 700 points where every query points, and its value is far from all others: a query sees it iff it lies in
    its window — at the window's first position yes, one further back no — in a prompt, in portions that end at page borders
    and in single decoded tokens.  Scores are capped, and the values are turned: the reader sees the planted value turned by the
    distance."""
    from tgis_amd import native

    H, G, dk, dv = geom
    g = torch.Generator().manual_seed(window)
    n, planted = 700, 411
    u = torch.randn(G, dk, generator=g)
    q = u.repeat_interleave(H // G, 0)[None] + 0.05 * torch.randn(n, H, dk, generator=g)
    k, v = torch.randn(n, G, dk, generator=g) * 0.3, torch.randn(n, G, dv, generator=g)
    k[planted] = u
    v[planted] = 50.0
    vfreq = ref.pair_frequencies(900.0, dv)
    pos = torch.arange(n)
    # the planted value as a reader at position i gets it
    seen = ref.turn_pairs(torch.full((n, 1, dv), 50.0, dtype=D), (planted - pos), vfreq)
    for pieces in ([700], [planted + window - 1, 1, 1, 1] + [n - planted - window - 2], [416, 32, 32, 220], [planted + 1] + [1] * (n - planted - 1)):
        got = _write_and_attend(native, gpu_device, dtype, q, k, v, 1.0, window, None, vfreq.float(), pieces, softcap=30.0).double().cpu().view(n, H, dv)
        share = (got * seen).sum(-1) / (seen * seen).sum(-1)  # the planted value's weight, about
        inside = (pos >= planted) & (pos - planted < window)
        assert float(share[inside].min()) > 0.9, (pieces[:3], float(share[inside].min()))
        assert float(share[~inside].abs().max()) < 0.1, (pieces[:3], float(share[~inside].abs().max()))
        assert float(share[planted + window - 1].min()) > 0.9 and float(share[planted + window].abs().max()) < 0.1


def test_the_sink_takes_its_share(gpu_device):
    """Keys that score zero against a sink of ln 5: with three visible keys the values' weights sum to 3 / 8, capped or not."""
    from tgis_amd import native

    n, v = 40, torch.ones(40, 1, 32)
    for cap in (0.0, 4.0):
        for dtype in DTYPES:
            got = _write_and_attend(native, gpu_device, dtype, torch.zeros(n, 2, 16), torch.randn(n, 1, 16), v, 1.0, 3, None, None, [37, 1, 2],
                                    sink=torch.log(torch.tensor([5.0, 1e-9])), softcap=cap).float().cpu().view(n, 2, 32)
            assert torch.allclose(got[2:, 0], torch.full((n - 2, 32), 3 / 8), atol=3e-3) and torch.allclose(got[2:, 1], torch.ones(n - 2, 32), atol=3e-3)
            assert torch.allclose(got[0, 0], torch.full((32,), 1 / 6), atol=3e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("q_rank,kv_rank", [(56, 48), (7, 11), (192, 256), (1100, 64)])
def test_latent_norm_and_cache_write(gpu_device, dtype, q_rank, kv_rank):
    """Both forms of the value write (inline on short steps, transposing on long ones) leave the same pages."""
    from tgis_amd import native

    g = torch.Generator().manual_seed(q_rank)
    dev, n = gpu_device, 600
    c_col = q_rank + 3
    down = torch.randn(n, c_col + kv_rank + 5, generator=g).to(dtype)
    qg, cg = 1 + 0.2 * torch.randn(q_rank, generator=g), 1 + 0.2 * torch.randn(kv_rank, generator=g)
    want_q = ref.rms_unit(down[:, :q_rank].double(), 1e-5) * qg.double()
    want_c = ref.rms_unit(down[:, c_col:c_col + kv_rank].double(), 1e-5) * cg.double()
    order = torch.randperm(20, generator=g)[:19]
    p = torch.arange(n)
    slots = (order[p // 32] * 32 + p % 32).to(torch.int32)
    tol = 1e-5 if dtype == torch.float32 else 0.01
    for pieces in ([600], [100, 1, 499]):
        kp, vp = torch.zeros(20, 1, 32 * kv_rank, dtype=dtype, device=dev), torch.zeros(20, 1, kv_rank * 32, dtype=dtype, device=dev)
        outs, at = [], 0
        for c in pieces:
            outs.append(native.latent_norm_write(down[at:at + c].to(dev).clone(), 0, q_rank, qg.to(dev), c_col, kv_rank, cg.to(dev), slots[at:at + c].to(dev), kp, vp, 1e-5))
            at += c
        assert float((torch.cat(outs).double().cpu() - want_q).abs().max()) <= tol * float(want_q.abs().max())
        K = kp.view(20, 32, kv_rank).double().cpu()[order][:, :, :].reshape(-1, kv_rank)[:n]
        V = vp.view(20, kv_rank, 32).transpose(1, 2).double().cpu()[order].reshape(-1, kv_rank)[:n]
        assert float((K - want_c).abs().max()) <= tol * float(want_c.abs().max()) and torch.equal(K, V)


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_attention_finds_a_far_token(gpu_device, dtype):
    """A model of two latent layers, the second on the first one's cache: the token at position 5 (and nothing else) has latents
    that the later queries ask for.  Its identity must be visible 600 positions later, in a prompt and in decoding."""
    H, dk, rk, W = 2, 16, 24, 32
    cfg = tiny.make_config([tiny.latent_layer(heads=H, dim=dk, vdim=16, kv_rank=rk, q_rank=16, scale=1.0, mlp=None),
                            tiny.latent_layer(heads=H, dim=dk, vdim=16, kv_rank=rk, q_rank=16, scale=1.0, kv_from=0, mlp=None)],
                           width=W, vocab=64, streams=2, scale=1.0)
    tensors = tiny.make_tensors(cfg, seed=5)
    # the queries of either layer carry a constant direction (every embedding has a large first channel), which the planted tokens'
    # latents answer: token 1 and token 2 share a large second channel and differ elsewhere
    e = torch.randn(64, W, generator=torch.Generator().manual_seed(1)) * 0.3
    e[:, 0], e[:, 1] = 3.0, 0.0
    e[1:3] *= 6.0
    e[1:3, 0], e[1:3, 1] = 3.0, 8.0
    tensors["embed"] = e.to(torch.bfloat16)
    for i in (0, 1):
        dq, uq, uk = torch.zeros(16, W), torch.zeros(H * dk, 16), torch.zeros(H * dk, rk)
        dq[:, 0] = 1.0
        uq[:, :] = 0.25
        uk[:, 0] = 0.4
        tensors[f"l{i}.mix.dq"], tensors[f"l{i}.mix.uq"], tensors[f"l{i}.mix.uk"] = (t.to(torch.bfloat16) for t in (dq, uq, uk))
        tensors[f"l{i}.mix.o"] = tensors[f"l{i}.mix.o"] * 8
    dkv = tensors["l0.mix.dkv"].float()
    dkv[:, :2] = 0.0
    dkv[0] = 0.0
    dkv[0, 1] = 1.0
    tensors["l0.mix.dkv"] = dkv.to(torch.bfloat16)
    model = ref.GopetarRef(cfg, tensors)
    g = torch.Generator().manual_seed(2)
    toks = torch.randint(3, 64, (620,), generator=g).tolist()
    lm = build_lm(cfg, tensors, dtype, pages=24)
    seen = []
    for planted in (1, 2):
        t = toks[:5] + [planted] + toks[6:]
        want = model.forward(t)
        with lm.context_manager():
            seq = lm.open_sequence()
            got = [lm.step_sequences([(seq, t[:600])])] + [lm.step_sequences([(seq, [x])]) for x in t[600:]]
            lm.close_sequence(seq)
        got = torch.cat(got).double().cpu()
        assert close(got, want, dtype), rel_err(got, want)
        seen.append(got)
    # the two prompts differ at position 5 only, and every later row shows which one it was
    assert float(row_errors(seen[0][:5], seen[1][:5]).max()) < 1e-6
    assert float(row_errors(seen[0][560:], seen[1][560:]).min()) > 2 * TOL[torch.bfloat16]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [5, 37, 600])
@pytest.mark.parametrize("E,k,W,ff,shared", [(6, 2, 72, 40, 56), (12, 4, 64, 96, None), (3, 3, 37, 21, 13), (1, 1, 40, 16, 40), (4, 2, 96, 160, 32)])
def test_mixture_of_clamped_units(gpu_device, dtype, T, E, k, W, ff, shared):
    """Routed and shared clamped units (gates and ups on both sides of their limits), summed by the combine launch and left to the
    consumer."""
    from tgis_amd import native
    from tgis_amd.utils.mixers import RoutedExperts
    from tgis_amd.utils.weights import DictWeights

    class _One:
        def size(self):
            return 1

        def rank(self):
            return 0

    cfg = tiny.make_config([tiny.latent_layer(mlp=tiny.moe_mlp(experts=E, top=k, ff=ff, limit=0.8, shared_ff=shared, shared_limit=0.4))], width=W)
    tensors = tiny.make_tensors(cfg, seed=E)
    p = {n[len("l0.mlp."):]: v.double() for n, v in tensors.items() if n.startswith("l0.mlp.")}
    g = torch.Generator().manual_seed(T)
    h = torch.randn(T, W, generator=g).to(dtype)
    logits = h.double() @ p["router"].T
    if k < E:  # rows near a routing tie are not compared
        b = logits.sort(-1, descending=True).values
        sure = (b[:, k - 1] - b[:, k]) > 1e-3
    else:
        sure = torch.ones(T, dtype=torch.bool)
    want = ref.mixture(h.double(), p, cfg["layers"][0]["mlp"])
    w = DictWeights(tensors, device=gpu_device, dtype=dtype, process_group=_One())
    ex = RoutedExperts(w, "l0.mlp", experts=E, top=k, shared=bool(shared), softmax_top=True, weight_on_input=False, clamp=(1.702, 0.8),
                       shared_clamp=(1.702, 0.4) if shared else None)
    got = ex(h.to(gpu_device)).double().cpu()
    tol = 2e-5 if dtype == torch.float32 else 0.03
    assert float((got - want)[sure].abs().max()) <= tol * float(want.abs().max())
    rows = ex(h.to(gpu_device), defer=True)
    one = torch.tensor([0.0, 1.0], device=gpu_device)  # mix 0, out 1: the stream becomes the result
    nxt = torch.tensor([1.0, 1.0], device=gpu_device)
    X, _ = native.hyper_update(torch.randn(T, 1, W, device=gpu_device), rows, one, nxt, 1e-5, dtype)
    assert float((X[:, 0].double().cpu() - want)[sure].abs().max()) <= tol * float(want.abs().max())


@pytest.mark.parametrize("dtype", [torch.float16, torch.bfloat16])
@pytest.mark.parametrize("N,K", [(64, 32), (200, 96), (320, 512), (1024, 160)])
@pytest.mark.parametrize("glu", [0, 1, 2])
def test_grouped_products_in_tiles_of_128_rows(gpu_device, dtype, N, K, glu):
    """Pairs spread unevenly over seven experts, one without any: gathered rows with a weight on the input and rows in place, every
    activation, against plain products; the 32-row tiles must agree."""
    from tgis_amd import native

    g = torch.Generator().manual_seed(N + K + glu)
    dev, T, k, E = gpu_device, 450, 2, 7
    share = torch.tensor([0.4, 0.02, 0.2, 0.0, 0.1, 0.18, 0.1])
    idx = torch.stack([torch.multinomial(share, k, generator=g) for _ in range(T)]).to(torch.int32)
    h = torch.randn(T, K, generator=g).to(dtype)
    w = (torch.randn(E, 2 * N if glu else N, K, generator=g) * K ** -0.5).to(dtype)
    scale = torch.rand(T * k, generator=g) + 0.5
    clamp = (1.702, 0.6) if glu == 2 else None

    def act(z):
        if not glu:
            return z
        a, b = z[..., :N], z[..., N:]
        if glu == 1:
            return ref.silu(a) * b
        a, b = a.clamp(max=0.6), b.clamp(-0.6, 0.6)
        return a * torch.sigmoid(1.702 * a) * (b + 1)

    rows = h.double().repeat_interleave(k, 0)
    flat = idx.view(-1).long()
    prod = lambda x: act(torch.stack([x[i] @ w[flat[i]].double().T for i in range(T * k)]))
    want, want_scaled = prod(rows), prod((rows * scale.double()[:, None]).to(dtype).double())
    assert native.moe_tile_rows(T * k, E, 32, 32, dtype) == 128 and native.moe_tile_rows(T * k, E, 32, 40, dtype) == 32
    tol = 0.02 if dtype == torch.bfloat16 else 0.003
    for tile in (128, 32):
        srt, te, pos, nt = native.moe_align(idx.to(dev), E, tile)
        cap = srt.shape[0]
        kw = dict(clamp=clamp, tile_rows=tile)
        wi = native.MoeWeight(w.to(dev), glu=bool(glu))
        got = native.moe_gemm(h.to(dev), wi, te, nt, cap, sorted_=srt, pair_div=k, **kw)
        got_s = native.moe_gemm(h.to(dev), wi, te, nt, cap, sorted_=srt, pair_div=k, pair_scale=scale.to(dev), **kw)
        placed = torch.zeros(cap, K, dtype=dtype, device=dev)
        placed[pos.long()] = h.to(dev).repeat_interleave(k, 0)
        got_p = native.moe_gemm(placed, wi, te, nt, cap, **kw)
        got_m = native.moe_gemm(placed, wi, te, nt, cap, sorted_=srt, pair_div=0, **kw)
        for out, ref_out in ((got, want), (got_s, want_scaled), (got_p, want), (got_m, want)):
            o = out[pos.long()].double().cpu()
            assert float((o - ref_out).abs().max()) <= tol * float(ref_out.abs().max()), tile


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
    model = ref.GopetarRef(cfg, tensors)
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

    layers = [tiny.pair_layer(left=tiny.attention_part(heads=8, kv_heads=4, dim=16, vdim=32, scale=0.25, window=20, rot_dims=4), width=40,
                              mlp=tiny.moe_mlp(experts=4, top=2, ff=32)),
              tiny.latent_layer(heads=2, dim=16, vdim=32, kv_rank=32, q_rank=24, mlp=tiny.moe_mlp(experts=5, top=3, ff=24, shared_ff=None)),
              tiny.latent_layer(heads=4, dim=8, vdim=8, kv_rank=32, q_rank=16, kv_from=1, mlp=None)]
    cfg = tiny.make_config(layers, width=64, vocab=70, eps=1e-6, streams=2)
    tensors = tiny.make_tensors(cfg, seed=11)
    model_dir = tmp_path / "model"
    model_dir.mkdir()
    (model_dir / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in tensors.items()}, str(model_dir / "model.safetensors"))
    prompts = {"a": rand_tokens(60, cfg, tensors, 1), "b": rand_tokens(33, cfg, tensors, 2), "c": rand_tokens(64, cfg, tensors, 3), "d": rand_tokens(40, cfg, tensors, 4)}
    model = ref.GopetarRef(cfg, tensors)
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
