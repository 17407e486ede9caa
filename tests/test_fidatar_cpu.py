"""CPU: what the Fidatar family needs and a GPU does not — the oracle's own consistency (whole sequence == token by token ==
portions through its explicit state), hand-checkable instances of its equations, the frequency scaling of the product, the config
reader, model dispatch by config.json, and the family's build units."""
import json
import math
import os

import pytest
import torch

from oracle import fidatar_ref as ref
from oracle import fidatar_tiny as tiny

D = torch.float64


def rand_tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def test_oracle_portions_equal_whole():
    cfg = tiny.make_config(tiny.standard_layers())
    model = ref.FidatarRef(cfg, tiny.make_tensors(cfg, seed=1))
    toks = rand_tokens(61, cfg["vocab"], 0)
    whole = model.forward(toks)
    for cuts in ([1] * 61, [2] * 30 + [1], [17, 1, 43], [47, 2, 12], [60, 1]):
        st, outs, at = model.new_state(), [], 0
        for n in cuts:
            outs.append(model.advance(st, toks[at:at + n]))
            at += n
        assert torch.allclose(torch.cat(outs), whole, atol=1e-9, rtol=1e-9), cuts


def test_oracle_attention_against_definitions():
    # blocks of 4: position 9 sees 8 and 9, position 7 sees 4 .. 7; 1 joins the denominator
    K, V = torch.zeros(12, 1, 1, dtype=D), torch.arange(12, dtype=D).view(12, 1, 1)
    o = ref.attend_in_blocks(torch.zeros(2, 1, 1, dtype=D), K, V, torch.tensor([9, 7]), 1.0, block=4)
    assert abs(float(o[0]) - (8 + 9) / 3) < 1e-12 and abs(float(o[1]) - (4 + 5 + 6 + 7) / 5) < 1e-12
    # large scores of either sign: the 1 is not scaled with them
    q, K, V = torch.ones(1, 1, 1, dtype=D), torch.tensor([[[-3.0]], [[2.0]]], dtype=D), torch.tensor([[[1.0]], [[2.0]]], dtype=D)
    o = ref.attend_in_blocks(q, K, V, torch.tensor([1]), 2.0)
    e = [math.exp(-6.0), math.exp(4.0)]
    assert abs(float(o) - (e[0] + 2 * e[1]) / (1 + e[0] + e[1])) < 1e-12
    # channel i turns with channel i + n, both grow by the factor, the rest passes
    x = torch.tensor([[[1.0, 2.0, 0.0, 0.0, 5.0]]], dtype=D)
    y = ref.turn_halves(x, torch.tensor([2]), torch.tensor([0.3, 0.05], dtype=D), amp=2.0)
    want = [2 * math.cos(0.6), 4 * math.cos(0.1), 2 * math.sin(0.6), 4 * math.sin(0.1), 5.0]
    assert torch.allclose(y[0, 0], torch.tensor(want, dtype=D))


def test_oracle_frequencies_against_definitions():
    # base 10000, 4 pairs; a pair turns 2 pi f original-independent radians per token.  d(t) = 8 ln(o / (2 pi t)) / (2 ln 10000)
    o = 2 * math.pi * 100
    sc = {"factor": 4.0, "original": o, "fast": 100 / 10 ** 0.5, "slow": 100 / 10 ** 2.5}  # d = 4 * 0.5 / 4 = 0.5 and 4 * 2.5 / 4 = 2.5
    f, amp = ref.yarn_frequencies(10000.0, 8, sc)
    plain = [1.0, 0.1, 0.01, 0.001]
    ramp = [0.0, 1 / 3, 2 / 3, 1.0]  # floor(0.5) = 0 to ceil(2.5) = 3
    for i in range(4):
        assert abs(float(f[i]) - (plain[i] / 4 * ramp[i] + plain[i] * (1 - ramp[i]))) < 1e-15
    assert abs(amp - (0.1 * math.log(4.0) + 1)) < 1e-15
    assert ref.yarn_frequencies(10000.0, 8)[1] == 1.0
    # both ends of the ramp at the same pair: a step, not a division by zero
    f, _ = ref.yarn_frequencies(10000.0, 8, {"factor": 4.0, "original": o, "fast": 10.0, "slow": 10.0})
    assert torch.allclose(f, torch.tensor([1.0, 0.1, 0.0025, 0.00025], dtype=D)) or torch.allclose(f, torch.tensor([1.0, 0.025, 0.0025, 0.00025], dtype=D))


def test_oracle_matrix_memory_against_definitions():
    one = lambda *x: torch.tensor(x, dtype=D)
    S, n, m = torch.zeros(1, 1, 1, dtype=D), torch.zeros(1, 1, dtype=D), one(0.0)
    # m starts at 0: an input gate of -2 leaves it there when nothing is forgotten, and the floor of the denominator is e^0 = 1
    S, n, m, o = ref.matrix_memory_step(S, n, m, torch.full((1, 1), 3.0, dtype=D), torch.full((1, 1), 2.0, dtype=D), torch.full((1, 1), 5.0, dtype=D), one(-2.0), one(-0.0))
    w = math.exp(-2.0)
    assert float(m) == 0.0 and abs(float(S) - 10 * w) < 1e-12 and abs(float(n) - 2 * w) < 1e-12
    assert abs(float(o) - 30 * w / (max(6 * w, 1.0) + 1e-6)) < 1e-12
    # a larger input gate lifts the maximum: the old state shrinks by e^(f + m - m')
    S2, n2, m2, o2 = ref.matrix_memory_step(S, n, m, torch.full((1, 1), 1.0, dtype=D), torch.full((1, 1), 1.0, dtype=D), torch.full((1, 1), -1.0, dtype=D), one(3.0), one(-0.5))
    k = math.exp(-0.5 - 3.0)
    assert float(m2) == 3.0 and abs(float(S2) - (10 * w * k - 1)) < 1e-12 and abs(float(n2) - (2 * w * k + 1)) < 1e-12
    assert abs(float(o2) - float(S2) / (max(float(n2), math.exp(-3.0)) + 1e-6)) < 1e-12


def test_oracle_routing_against_definitions():
    logit = lambda s: math.log(s / (1 - s))
    w = torch.tensor([[logit(s)] for s in (0.9, 0.1, 0.6, 0.5, 0.8, 0.2)], dtype=D)
    h = torch.ones(1, 1, dtype=D)
    # groups by their two best: 1.0, 1.1, 1.0; one kept: the best single expert is not among them
    idx, wt = ref.route(h, w, {"experts": 6, "top": 2, "scale": 2.0, "groups": {"count": 3, "keep": 1}})
    assert idx[0].tolist() == [2, 3] and torch.allclose(wt[0], torch.tensor([1.2, 1.0], dtype=D))
    idx, _ = ref.route(h, w, {"experts": 6, "top": 2})
    assert idx[0].tolist() == [0, 4]
    # two groups of three: 1.5 against 1.3
    idx, _ = ref.route(h, w, {"experts": 6, "top": 3, "groups": {"count": 2, "keep": 1}})
    assert idx[0].tolist() == [0, 2, 1]
    # groups of one
    idx, _ = ref.route(h, w, {"experts": 6, "top": 2, "groups": {"count": 6, "keep": 3}})
    assert idx[0].tolist() == [0, 4]
    assert ref.relu2(torch.tensor([-3.0, 2.0])).tolist() == [0.0, 4.0]


def test_oracle_norms_after_the_sum():
    """A layer whose sublayers add nothing: the stream is normed twice, the first norm's scale is gone, c does not matter."""
    cfg = tiny.make_config([tiny.mlstm_layer(mlp=tiny.dense_mlp())], softcap=None, alpha=2.0)
    t = tiny.make_tensors(cfg, seed=0)
    for n in ("l0.mix.o", "l0.mlp.down"):
        t[n] = torch.zeros_like(t[n])
    trace = []
    ref.FidatarRef(cfg, t).forward([5, 7], trace)
    x = t["embed"].double()[[5, 7]]
    want = ref.rms_unit(ref.rms_unit(x, 1e-6) * t["l0.norm1"].double(), 1e-6) * t["l0.norm2"].double()
    assert torch.allclose(trace[0], want, atol=1e-4)


def test_scaled_frequencies_of_the_product():
    from tgis_amd.utils.mixers import yarn_inverse_frequencies

    kinds = set()
    for base, dims, sc in ((5000.0, 16, tiny.SCALING), (500000.0, 64, {"factor": 8.0, "original": 8192, "fast": 32.0, "slow": 1.0}),
                           (100.0, 10, {"factor": 2.0, "original": 50, "fast": 2.0, "slow": 2.0}), (10000.0, 32, None), (7.0, 2, tiny.SCALING),
                           (10000.0, 128, {"factor": 40.0, "original": 4096, "fast": 32.0, "slow": 0.01}), (1000.0, 6, {"factor": 3.0, "original": 4, "fast": 64.0, "slow": 1.0})):
        want, amp = ref.yarn_frequencies(base, dims, sc)
        got, a = yarn_inverse_frequencies(base, dims, sc, "cpu")
        assert got.dtype == torch.float32 and torch.allclose(got.double(), want, rtol=1e-7, atol=0) and abs(a - amp) < 1e-12
        if sc:
            r = want / ref.yarn_frequencies(base, dims)[0] * sc["factor"]
            kinds |= {"kept"} if (r > sc["factor"] - 1e-9).any() else set()
            kinds |= {"divided"} if (r < 1 + 1e-9).any() else set()
            kinds |= {"between"} if ((r > 1 + 1e-6) & (r < sc["factor"] - 1e-6)).any() else set()
    assert kinds == {"kept", "divided", "between"}


def test_config_reader_and_dispatch(tmp_path):
    from tgis_amd.models import config_model_type
    from tgis_amd.models.custom_modeling.flash_fidatar_modeling import FidatarConfig

    cfg = tiny.make_config(tiny.standard_layers(), width=64, vocab=96, eps=1e-5, scale=3.0, alpha=2.5, softcap=11.0)
    c = FidatarConfig(**cfg)
    assert (c.width, c.vocab, c.eps, c.embedding_scale, c.postln_alpha, c.logit_softcap) == (64, 96, 1e-5, 3.0, 2.5, 11.0)
    assert c.hidden_size == 64 and c.vocab_size == 96 and c.num_hidden_layers == 5 and c.model_type == "fidatar"
    assert config_model_type(cfg) == "fidatar"
    assert FidatarConfig(**{k: v for k, v in cfg.items() if k != "logit_softcap"}).logit_softcap == 0.0
    with pytest.raises(ValueError):
        FidatarConfig(**{**cfg, "layers": [{"type": "conv", "mixer": {}, "mlp": None}]})
    with pytest.raises(ValueError):
        FidatarConfig(**{**cfg, "layers": [tiny.mlstm_layer(mlp={"kind": "gated"})]})
    from tgis_amd.inference_engine.engine import BaseInferenceEngine

    (tmp_path / "config.json").write_text(json.dumps(cfg))
    loaded = BaseInferenceEngine._load_config(str(tmp_path))
    assert isinstance(loaded, FidatarConfig) and loaded.layers == cfg["layers"] and loaded.to_dict() == cfg
    if not torch.cuda.is_available():
        from tgis_amd.models import get_model

        with pytest.raises(NotImplementedError):
            get_model(str(tmp_path), None, "tgis_native", "bfloat16", None, None)


def test_build_units_and_slot_shapes():
    from tgis_amd import buildlib
    from tgis_amd.utils.state_cache import RecurrentStateCache

    for u in buildlib.FAMILY_UNITS["fidatar"]:
        assert os.path.exists(os.path.join(buildlib.CSRC, u + ".hip")), u
    st = RecurrentStateCache([None, {"matrix": (3, 24, 40), "memory": (3, 25)}], width=72, num_slots=2, device="cpu")
    assert st.state[0] is None and st.state[1].shape == (3, 3, 24, 40) and st.shift[1].shape == (3, 3, 25)
