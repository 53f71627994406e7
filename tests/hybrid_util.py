"""Small configurations and random weights for the hybrid decoders' tests, and the comparison with the plain oracle."""
import torch

from oracle import hybrid_ref as ref
from trimkv_amd.fusitar import FusitarConfig, FusitarForCausalLM

DEV = "cuda:0"


def attention(heads=4, kv_heads=2, dim=24, vdim=40, size=9, keep_first=3, scale=None, mlp=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5 * 1.3,
                                           "mask": {"size": size, "keep_first": keep_first}}, "mlp": mlp}


def mlstm(heads=3, dim=40, vdim=24, gate_cap=7.0, mlp=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}, "mlp": mlp}


def moe(experts=6, top=2, ff=40, count=3, keep=2):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}}}


def config(layers, vocab=97, width=72, eps=2e-5, scale=3.0):
    return {"architecture": "Fusitar", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps}, "layers": layers}


def weights(cfg, seed=0):
    """Checkpoint tensors in bf16: unit-gain matrices, norms around one, gates and corrections that matter."""
    gen = torch.Generator().manual_seed(seed)
    rnd = lambda *s: torch.randn(*s, generator=gen)
    W = cfg["width"]
    out = {"embed": rnd(cfg["vocab"], W), "final.norm": 1 + 0.2 * rnd(W)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        out[f"l{i}.norm1"] = 1 + 0.2 * rnd(W)
        H, D, Dv = m["heads"], m["dim"], m["vdim"]
        G = m.get("kv_heads", H)
        mats = {"q": (H * D, W), "k": (G * D, W), "v": (G * Dv, W), "g": (H * Dv, W), "o": (W, H * Dv)}
        if layer["type"] == "attention":
            out[p + "q.norm"], out[p + "k.norm"] = 1.5 + 0.3 * rnd(H * D), 1.5 + 0.3 * rnd(G * D)
        else:
            mats.update({"i": (H, W), "f": (H, W)})
            out[p + "i.b"], out[p + "f.b"] = rnd(H), 2 + 2 * rnd(H)
            out[p + "norm"] = 1 + 0.2 * rnd(H * Dv)
        if layer["mlp"] is not None:
            out[f"l{i}.norm2"] = 1 + 0.2 * rnd(W)
            r, ff = layer["mlp"]["router"], layer["mlp"]["expert"]["ff"]
            q = f"l{i}.mlp."
            out[q + "router"] = 2 * rnd(r["experts"], W) * W ** -0.5
            out[q + "correction"] = 0.3 * rnd(r["experts"]) - 0.6          # choice scores of both signs
            for e in range(r["experts"]):
                out[f"{q}e{e}.up"], out[f"{q}e{e}.down"] = rnd(ff, W) * W ** -0.5, rnd(W, ff) * ff ** -0.5
        for name, shape in mats.items():
            out[p + name] = rnd(*shape) * shape[1] ** -0.5
    return {k: v.to(torch.bfloat16) for k, v in out.items()}


def build(cfg, w, dtype):
    model = FusitarForCausalLM(FusitarConfig.from_dict(cfg), dtype)
    model.load_tensors(w)
    return model.to(DEV).eval()


def tokens(cfg, n, seed=1):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def oracle(cfg, w, toks):
    return ref.forward(cfg, w, toks)


def row_error(got, want):
    """Root mean square difference per row over the spread of the wanted rows."""
    d = got.detach().double().cpu() - want
    return (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std()


TOL = {torch.float32: 3e-5, torch.bfloat16: 0.06}


def assert_rows(got, want, dtype, what=""):
    err = row_error(got, want)
    # a router that is close to a tie may choose otherwise in bf16: one row in ten may be further off
    allowed = 0 if dtype == torch.float32 else max(1, len(err) // 10)
    over = int((err > TOL[dtype]).sum())
    assert over <= allowed, f"{what}: {over} of {len(err)} rows off, worst {float(err.max()):.3e} at {int(err.argmax())}"
