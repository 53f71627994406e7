"""Small configurations and random weights for the Siterax tests."""
import torch

from oracle import siterax_ref as ref
from trimkv_amd.siterax import SiteraxConfig, SiteraxForCausalLM
from tests.hybrid_util import DEV


def attention(heads=4, kv_heads=2, dim=24, vdim=40, size=9, rot_dims=None, base=500.0, factor=1.5, scale=None, ff=56):
    return {"type": "attention", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5 * 1.2, "mask": {"size": size},
                      "rot": {"base": base, "dims": rot_dims or dim, "scaling": {"factor": factor}}}}


def config(layers, loop=None, vocab=97, width=72, eps=3e-5, mult=0.6, cap=9.0):
    return {"architecture": "Siterax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult, "logit_softcap": cap, "loop": loop, "layers": layers}


# sizes that differ from layer to layer, loops at the start, in the middle and up to the end, passes of several counts, heads and
# rotations with and without padding, layers without a feed-forward
CONFIGS = {
    "looped_middle": config([attention(), attention(heads=6, kv_heads=1, dim=32, vdim=16, size=21, rot_dims=16, base=80.0, factor=3.0, ff=None),
                             attention(heads=2, kv_heads=2, dim=16, vdim=24, size=5, ff=24), attention(size=40, ff=None)], {"start": 1, "stop": 3, "times": 3}),
    "looped_to_the_end": config([attention(heads=3, kv_heads=3, dim=20, vdim=12, size=1, rot_dims=6, factor=1.0, ff=33), attention(heads=8, kv_heads=1, dim=64, vdim=64, size=70, ff=128)],
                                {"start": 0, "stop": 2, "times": 2}, vocab=130, width=100, eps=1e-6, mult=1.0, cap=4.0),
    "single_pass": config([attention(heads=5, kv_heads=1, dim=48, vdim=56, size=33, rot_dims=32, base=10000.0, factor=8.0, ff=200)], {"start": 0, "stop": 1, "times": 1}, vocab=51, width=192, mult=0.35),
    "one_layer_often": config([attention(heads=2, kv_heads=1, dim=128, vdim=96, size=64, rot_dims=64, ff=40), attention(heads=4, kv_heads=4, dim=8, vdim=8, size=300, ff=None)],
                              {"start": 1, "stop": 2, "times": 4}, width=61),
    "no_loop": config([attention(heads=9, kv_heads=3, dim=40, vdim=8, size=17, rot_dims=40), attention()], cap=30.0),
}


def weights(cfg, seed=0):
    """Checkpoint tensors in bf16: unit-gain matrices, norms around one and more than that for q and k, biases and caps that matter."""
    gen = torch.Generator().manual_seed(seed)
    rnd = lambda *s: torch.randn(*s, generator=gen)
    W = cfg["width"]
    out = {"embed": rnd(cfg["vocab"], W), "final.norm": 1 + 0.2 * rnd(W), "head": 5 * rnd(cfg["vocab"], W) * W ** -0.5}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        H, G, D, Dv = (m[k] for k in ("heads", "kv_heads", "dim", "vdim"))
        mats = {p + "q": (H * D, W), p + "k": (G * D, W), p + "v": (G * Dv, W), p + "g": (H, W), p + "o": (W, H * Dv)}
        out.update({p + "q.b": 0.7 * rnd(H * D), p + "k.b": 0.7 * rnd(G * D), p + "v.b": 0.5 * rnd(G * Dv), p + "q.norm": 1.5 + 0.3 * rnd(D), p + "k.norm": 1.5 + 0.3 * rnd(D)})
        norms = ["norm1", "norm1b"]
        if layer["mlp"] is not None:
            ff, q = layer["mlp"]["ff"], f"l{i}.mlp."
            mats.update({q + "gate": (ff, W), q + "up": (ff, W), q + "down": (W, ff)})
            norms += ["norm2", "norm2b"]
        out.update({f"l{i}.{n}": 1 + 0.2 * rnd(W) for n in norms})
        out.update({n: rnd(*s) * s[1] ** -0.5 for n, s in mats.items()})
    return {k: v.to(torch.bfloat16) for k, v in out.items()}


def build(cfg, w, dtype):
    model = SiteraxForCausalLM(SiteraxConfig.from_dict(cfg), dtype)
    model.load_tensors(w)
    return model.to(DEV).eval()


def oracle(cfg, w, toks, layers_out=None):
    return ref.forward(cfg, w, toks, layers_out=layers_out)
