"""CPU checks of the hybrid decoders: ABI of their libraries, configuration and registry, loading, refusal to run without a
GPU, and the oracle's own mechanisms on cases small enough to work out by hand."""
import ctypes
import json
import math
import os
import re

import pytest
import torch
from safetensors.torch import save_file

from oracle import hybrid_ref as ref
from trimkv_amd import _lib, registry
from trimkv_amd.hybrid_ops import pack_matrix, unpack_matrix
from trimkv_amd.fusitar import FusitarConfig, FusitarForCausalLM
from tests.hybrid_util import attention, config, mlstm, moe, weights

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TEXT = re.sub(r"/\*.*?\*/", "", open(os.path.join(ROOT, "include", "trimkv_hybrid.h")).read(), flags=re.S)


def test_header_binding_and_library_agree():
    declared = sorted(set(re.findall(r"\b(trimkv_[a-z0-9_]+)\s*\(", TEXT)))
    assert sorted(n for sig in _lib.HYBRID_SIGNATURES.values() for n in sig) == declared
    for lib, name, argtypes in ((ctypes.CDLL(_lib.HYBRID_LIB_PATHS[l]), n, a) for l, sig in _lib.HYBRID_SIGNATURES.items() for n, (_, a) in sig.items()):
        assert hasattr(lib, name), name
        params = re.search(r"\b%s\s*\(([^;]*?)\)\s*;" % name, TEXT, flags=re.S).group(1).strip()
        want = [] if params in ("", "void") else [p.strip() for p in params.split(",")]
        kinds = [_lib.C.c_void_p if "*" in p else _lib.C.c_int64 if p.startswith("int64_t") else _lib.C.c_float if p.startswith("float") else _lib.C.c_int for p in want]
        assert kinds == argtypes, name


def test_bad_arguments_are_refused_without_a_launch():
    lib = _lib.load_hybrid()
    one = ctypes.c_void_p(16)
    embed = lambda ids=one, xh=None, norm=None, dt=_lib.F32: lib.trimkv_embed_scaled(ids, one, 1.0, one, xh, norm, 1e-6, 0, 1, 4, 8, 64, dt, None)
    assert embed(ids=None) == -1 and embed(norm=one) == -1 and embed(dt=_lib.F16) == -3
    assert lib.trimkv_residual_norm(one, 64, None, 1, one, one, 1.0, None, one, 1, 64, 64, 1e-6, _lib.BF16, None) == -1      # a norm with nowhere to go
    heads = lambda H=4, D=16, rot=8, table=one, kw=one: lib.trimkv_qkv_heads(one, 256, 0, 64, 80, None, one, kw, 1e-6, table, rot, H, 1, D, D, D, D, one, one, one, None, None, 0, 0, 1, _lib.BF16, None)
    assert heads(H=0) == -2 and heads(rot=18) == -2 and heads(rot=7) == -2 and heads(table=None) == -1 and heads(kw=None) == -1
    assert lib.trimkv_rotary_table(one, one, one, one, one, 1, 1, 7, None) == -2 and lib.trimkv_rotary_table(None, one, one, one, one, 1, 1, 8, None) == -1
    assert lib.trimkv_silu_gate(one, one, 4, one, 1, 8, _lib.BF16, None) == -2 and lib.trimkv_soft_cap(one, one, 4, 0.0, _lib.BF16, None) == -2
    assert lib.trimkv_linear_f32(one, 64, one, 64, one, 1, 3, 62, _lib.F32, None) == -2
    assert b"bad sizes" in lib.trimkv_hybrid_last_error()
    win = lambda H=4, G=2, D=16, Dp=16, keep=1, size=4, dt=_lib.BF16: lib.trimkv_window_decode(one, one, one, one, one, one, 64, one, 1, H, G, D, D, Dp, Dp, keep, size, 1.0, 0, 0, 1, None, dt, None)
    assert win(H=5) == -2 and win(Dp=12, D=12) == -2 and win(size=0) == -2 and win(keep=-1) == -2 and win(D=520, Dp=520) == -6 and win(dt=7) == -3
    assert lib.trimkv_window_decode(one, one, one, one, one, one, 64, one, 1, 4, 2, 16, 16, 16, 16, 1, 4, 1.0, 0, 0, 3, None, _lib.BF16, None) == -5
    recurrent, routed = _lib.load_hybrid("mlstm"), _lib.load_hybrid("moe")
    assert routed.trimkv_moe_route(one, one, one, one, 1, 8, 5, 2, 1, None) == -2          # one open group of four cannot give five
    assert routed.trimkv_moe_route(one, one, one, one, 1, 9, 2, 2, 1, None) == -2
    assert routed.trimkv_moe_gemm(one, 64, one, one, 64, one, one, one, 4, 2, 16, 1, 64, 64, 64, 1, _lib.BF16, None) == -2
    assert recurrent.trimkv_mlstm(one, 64, 0, 8, 16, one, one, one, 1.0, one, one, one, one, one, one, 1, 1, 1, 513, 8, 1, 1.0, None, _lib.F32, None) == -6
    assert lib.trimkv_window_decode_splits(64, 8, 4096) >= 1 and lib.trimkv_window_decode_splits(1, 1, 64) == 1
    assert recurrent.trimkv_mlstm_workspace(1, 1, 4, 64, 64, _lib.BF16) == 0


GOOD = config([attention(mlp=moe()), mlstm()])


def test_configuration_is_checked():
    cfg = FusitarConfig.from_dict(GOOD)
    assert (cfg.vocab_size, cfg.hidden_size, cfg.num_hidden_layers, cfg.norm_eps) == (97, 72, 2, 2e-5)
    for layer, text in ((attention(heads=5), "do not divide"), (dict(attention(), type="other"), "unknown mixer"), (attention(size=0), "bad window"),
                        (attention(mlp=moe(experts=7)), "cannot choose"), (attention(mlp=moe(top=5)), "cannot choose"), (attention(mlp=dict(moe(), kind="x")), "unknown feed-forward"),
                        ({"type": "mlstm", "mixer": {"heads": 1, "dim": 8, "vdim": 8}, "mlp": None}, "lacks")):
        with pytest.raises(ValueError, match=text):
            FusitarConfig.from_dict(dict(GOOD, layers=[layer]))


def test_registry_finds_every_family():
    assert registry.model_class(GOOD) is FusitarForCausalLM
    for name, (module, cls) in registry.MODELS.items():
        assert registry.model_class({"architectures": [name]}).__name__ == cls
    with pytest.raises(ValueError, match="no model for architecture"):
        registry.model_class({"architecture": "Nothing"})


def test_loading_fills_every_parameter_and_refuses_what_does_not_fit(tmp_path):
    w = weights(GOOD)
    (tmp_path / "config.json").write_text(json.dumps(GOOD))
    save_file(w, str(tmp_path / "model.safetensors"))
    model = registry.from_pretrained(str(tmp_path), torch_dtype=torch.float32)
    for name, t in model.tensors().items():
        assert torch.equal(t.value() if hasattr(t, "value") else t, w[name].float()), name
    # padding stays zero: kernels read it
    up, down = (unpack_matrix(m.data) for m in (model.model.layers[0].mlp.up, model.model.layers[0].mlp.down))
    assert up.shape == (6, 64, 128) and not up[:, 40:].any() and not up[:, :, 72:].any() and not down[:, 72:].any() and not down[:, :, 40:].any()
    # block (n / 32, k / 16): k 0..7 of its 32 outputs, then k 8..15
    m = torch.arange(64 * 128).view(64, 128)
    assert pack_matrix(m)[1, 3, 1, 5].tolist() == m[37, 56:64].tolist() and torch.equal(unpack_matrix(pack_matrix(m)), m)
    for change in (lambda d: d.pop("l1.mix.f.b"), lambda d: d.update(extra=torch.zeros(1)), lambda d: d.update({"l0.norm1": torch.zeros(71)})):
        bad = dict(w)
        change(bad)
        with pytest.raises(ValueError):
            model.load_tensors(bad)
    with pytest.raises(ValueError, match="bfloat16 or float32"):
        FusitarForCausalLM(FusitarConfig.from_dict(GOOD), torch.float16)


def test_no_cpu_path():
    model = FusitarForCausalLM(FusitarConfig.from_dict(GOOD))
    with pytest.raises(_lib.TrimKVLibraryError, match="GPU only"):
        model(torch.tensor([[1, 2]]))
    with pytest.raises(_lib.TrimKVLibraryError, match="GPU only"):
        model.new_cache()


# ---- the oracle on cases worked out by hand --------------------------------------------------------------
def test_oracle_window():
    seen = [[j for j in range(8) if ref.window_visible(i, j, 3, 2)] for i in range(8)]
    assert seen[0] == [0] and seen[3] == [0, 1, 2, 3] and seen[7] == [0, 1, 5, 6, 7]
    T = 8
    q = torch.zeros(T, 1, 1, dtype=torch.float64)
    v = torch.arange(T, dtype=torch.float64).view(T, 1, 1)
    out = ref.window_attention(q, q, v, 1.0, 3, 2).flatten()
    assert out.tolist() == pytest.approx([sum(s) / len(s) for s in seen])
    # sensitive to a window and to a kept prefix that are one off
    assert not torch.allclose(out, ref.window_attention(q, q, v, 1.0, 4, 2).flatten()) and not torch.allclose(out, ref.window_attention(q, q, v, 1.0, 3, 1).flatten())


def test_oracle_mlstm_first_steps():
    one = torch.ones(1, 1, 1, dtype=torch.float64)
    li, lf = torch.tensor([[math.log(0.5)], [math.log(3.0)]], dtype=torch.float64), torch.tensor([[math.log(0.25)], [math.log(0.5)]], dtype=torch.float64)
    out, (S, n, m) = ref.mlstm_scan(torch.cat([one, one]), torch.cat([one, 2 * one]), torch.cat([4 * one, 5 * one]), li, lf)
    # unscaled: S1 = 0.5 * 4, n1 = 0.5; m1 = max(log .25 + 0, log .5) = log .5, so S = 4, n = 1, floor exp(-m1) = 2
    assert out[0].item() == pytest.approx(4 / (2 + 1e-6))
    # S2 = 0.5 * 2 + 3 * 2 * 5 = 31, n2 = 0.25 + 6 = 6.25, m2 = log 3
    assert m.item() == pytest.approx(math.log(3)) and S.item() == pytest.approx(31 / 3) and n.item() == pytest.approx(6.25 / 3)
    assert out[1].item() == pytest.approx((31 / 3) / (6.25 / 3 + 1e-6))
    # the running maximum starts at 0: a first token with a tiny input gate is scaled down, not normalised away
    out, (S, _, m) = ref.mlstm_scan(one, one, one, torch.tensor([[-9.0]], dtype=torch.float64), torch.tensor([[-1.0]], dtype=torch.float64))
    assert m.item() == -1.0 and S.item() == pytest.approx(math.exp(-8.0))


def test_oracle_router_by_hand():
    z = torch.tensor([[0.0, 0.0, 2.0, -9.0, 1.0, 1.0]], dtype=torch.float64)
    corr = torch.tensor([-0.1, -0.1, -0.9, 0.0, -0.7, -0.7], dtype=torch.float64)
    s = torch.sigmoid(z[0])
    ids, w = ref.choose_experts(z, corr, 2, 3, 1)                 # groups (0, 1), (2, 3), (4, 5); the first has the largest sum
    assert sorted(ids[0].tolist()) == [0, 1] and torch.allclose(w, s[ids])
    # all choice scores negative: closed groups must stay closed
    ids, _ = ref.choose_experts(z, corr - 5.0, 2, 3, 1)
    assert sorted(ids[0].tolist()) == [0, 1]


def test_oracle_norm_has_eps_inside_the_root():
    x = torch.tensor([3.0, 4.0], dtype=torch.float64)
    assert torch.allclose(ref.rms(x, 12.5), x / 5.0)
