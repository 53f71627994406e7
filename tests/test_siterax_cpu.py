"""CPU checks of the Siterax decoder: configuration, registry, loading, order of layers, and the oracle's mechanisms on cases
small enough to work out by hand."""
import json
import math

import pytest
import torch
from safetensors.torch import save_file

from oracle import siterax_ref as ref
from trimkv_amd import _lib, registry
from trimkv_amd.hybrid_ops import RotarySpec
from trimkv_amd.siterax import SiteraxConfig, SiteraxForCausalLM
from tests.siterax_util import CONFIGS, attention, config, weights


def changed(layer, part, **values):
    return dict(layer, **{part: dict(layer[part], **values)})


def test_configuration_is_checked():
    good = CONFIGS["looped_middle"]
    cfg = SiteraxConfig.from_dict(good)
    assert (cfg.vocab_size, cfg.hidden_size, cfg.num_hidden_layers, cfg.norm_eps, cfg.residual_mult, cfg.logit_softcap) == (97, 72, 4, 3e-5, 0.6, 9.0)
    assert not cfg.tied_head and cfg.norms == "both"
    one = attention()
    no_rot = dict(one, mixer={k: v for k, v in one["mixer"].items() if k != "rot"})
    for layer, text in ((attention(heads=5), "do not divide"), (dict(one, type="mlstm"), "unknown mixer"), (attention(size=0), "bad window"), (attention(rot_dims=26), "bad rotation"),
                        (attention(rot_dims=5), "bad rotation"), (no_rot, "lacks"), (changed(one, "mlp", kind="moe"), "unknown feed-forward"), (changed(one, "mlp", ff=0), "bad feed-forward")):
        with pytest.raises(ValueError, match=text):
            SiteraxConfig.from_dict(dict(good, layers=[layer], loop=None))
    for loop in ({"start": 1, "stop": 1, "times": 2}, {"start": 0, "stop": 5, "times": 2}, {"start": 0, "stop": 2, "times": 0}):
        with pytest.raises(ValueError, match="loop"):
            SiteraxConfig.from_dict(dict(good, loop=loop))
    with pytest.raises(ValueError, match="logit_softcap"):
        SiteraxConfig.from_dict(dict(good, logit_softcap=0.0))


def test_order_of_layers():
    order = lambda n, loop: [tuple(r) for r in SiteraxConfig.from_dict(config([attention()] * n, loop)).layer_runs()]
    assert order(3, None) == [(0, False), (1, False), (2, False)]
    assert order(4, {"start": 1, "stop": 3, "times": 3}) == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    assert order(2, {"start": 1, "stop": 2, "times": 2}) == [(0, False), (1, False), (1, True)]
    for cfg in CONFIGS.values():
        assert [tuple(r) for r in SiteraxConfig.from_dict(cfg).layer_runs()] == ref.layer_order(len(cfg["layers"]), cfg["loop"])


def test_registry_and_libraries():
    cfg = CONFIGS["no_loop"]
    assert registry.model_class(cfg) is SiteraxForCausalLM
    assert SiteraxForCausalLM.libraries(SiteraxConfig.from_dict(cfg)) == ("hybrid",)      # neither recurrent layers nor experts to compile


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_loading_fills_every_parameter_and_refuses_what_does_not_fit(tmp_path, name):
    cfg = CONFIGS[name]
    w = weights(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    model = registry.from_pretrained(str(tmp_path), torch_dtype=torch.float32)
    assert sorted(model.tensors()) == sorted(w)
    for key, t in model.tensors().items():
        assert torch.equal(t, w[key].float()), key
    # every parameter is reached by some tensor; columns of alignment stay zero
    held = sum(t.numel() for t in model.tensors().values())
    spare = sum(l.mix.qkvg.weight.shape[0] - sum(n for _, n in l.mix.qkvg.offsets.values()) for l in model.model.layers)
    assert sum(p.numel() for p in model.parameters()) >= held and all(0 <= l.mix.qkvg.weight.shape[0] % 8 < 1 for l in model.model.layers) and spare < 8 * len(cfg["layers"])
    for l in model.model.layers:
        off, n = l.mix.qkvg.offsets["g"]
        assert not l.mix.qkvg.weight[off + n:].any() and not l.mix.bias[off:].any()
    for change in (lambda d: d.pop("l0.mix.k.b"), lambda d: d.update({"l0.mix.g.b": torch.zeros(1)}), lambda d: d.update({"l0.norm1b": torch.zeros(cfg["width"] + 1)}), lambda d: d.pop("head")):
        bad = dict(w)
        change(bad)
        with pytest.raises(ValueError):
            model.load_tensors(bad)


def test_no_cpu_path():
    model = SiteraxForCausalLM(SiteraxConfig.from_dict(CONFIGS["no_loop"]))
    with pytest.raises(_lib.TrimKVLibraryError, match="GPU only"):
        model(torch.tensor([[1, 2]]))


# ---- the oracle on cases worked out by hand --------------------------------------------------------------
def test_oracle_rotation():
    x = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 9.0]]], dtype=torch.float64).repeat(2, 1, 1)
    out = ref.rotate(x, 6, 4, 16.0, 2.0)                       # frequencies 1/2 and 1/8; pairs (0, 2) and (1, 3); feature 4 stays
    for t, p in enumerate((6, 7)):
        a, b = p / 2, p / 8
        want = [math.cos(a) - 3 * math.sin(a), 2 * math.cos(b) - 4 * math.sin(b), 3 * math.cos(a) + math.sin(a), 4 * math.cos(b) + 2 * math.sin(b), 9.0]
        assert out[t, 0].tolist() == pytest.approx(want)
    assert RotarySpec(4, 16.0, 2.0).frequencies().tolist() == pytest.approx([0.5, 0.125])


def test_oracle_sink_and_window():
    # equal scores of 0: n visible tokens and the sink share the weight
    T, z = 6, torch.zeros(6, 1, 1, dtype=torch.float64)
    v = torch.arange(1.0, 7.0, dtype=torch.float64).view(T, 1, 1)
    out = ref.sink_window_attention(z, z, v, 1.0, 3).flatten().tolist()
    assert out == pytest.approx([1 / 2, 3 / 3, 6 / 4, 9 / 4, 12 / 4, 15 / 4])
    w = ref.sink_weights(torch.tensor([math.log(2.0), -math.inf, math.log(5.0)], dtype=torch.float64))
    assert w.tolist() == pytest.approx([2 / 8, 0, 5 / 8])
    assert ref.sink_weights(torch.tensor([-800.0, -900.0], dtype=torch.float64)).tolist() == [0.0, 0.0]
    assert ref.sink_weights(torch.tensor([800.0, 700.0], dtype=torch.float64)).tolist() == pytest.approx([1.0, 0.0])


def test_oracle_gates():
    o = torch.ones(1, 2, 3, dtype=torch.float64)
    h = torch.tensor([[1.0]], dtype=torch.float64)
    gated = ref.head_gate(o, h, {"g": torch.tensor([[0.0], [math.log(3.0)]], dtype=torch.float64)})
    assert gated[0, 0].tolist() == pytest.approx([0.5] * 3) and gated[0, 1].tolist() == pytest.approx([0.75] * 3)
    w = {"gate": torch.tensor([[math.log(3.0)]], dtype=torch.float64), "up": torch.tensor([[2.0]], dtype=torch.float64), "down": torch.tensor([[10.0]], dtype=torch.float64)}
    assert ref.gated_mlp(h, w).item() == pytest.approx(math.log(3.0) * 0.75 * 2.0 * 10.0)


def test_oracle_layers_depend_on_what_they_should():
    """Leaving out a pass, the embedding between passes, a bias or the norm behind a sublayer changes the logits."""
    cfg = CONFIGS["looped_middle"]
    w, toks = weights(cfg), [3, 96, 0, 41, 41, 7, 12, 30, 5, 5, 5, 80]
    base = ref.forward(cfg, w, toks)
    seen = []
    ref.forward(cfg, w, toks, layers_out=seen)
    assert len(seen) == 8 and base.abs().max() < 9.0 and base.abs().max() > 4.0        # the cap bends them
    less = ref.forward(dict(cfg, loop=dict(cfg["loop"], times=2)), w, toks)
    flat = ref.forward(cfg, {k: torch.zeros_like(v) if k == "l2.mix.k.b" else v for k, v in w.items()}, toks)
    half = ref.forward(dict(cfg, residual_mult=0.3), w, toks)
    for other in (less, flat, half):
        assert (base - other).abs().max() > 0.05
