"""The mechanisms of the Siterax decoder one by one against the plain oracle (oracle/siterax_ref.py), on the GPU."""
import pytest
import torch

from oracle import siterax_ref as ref
from oracle.hybrid_ref import rms, soft_cap
from trimkv_amd import hybrid_ops as ops
from trimkv_amd.hybrid_cache import HybridCache
from tests.test_gpu_hybrid_ops import DEV, DTYPES, close, rnd

pytestmark = pytest.mark.gpu


# ---- row-wise steps ------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [40, 101, 1024, 4096, 5000])
def test_embedding_with_norm_and_added_again(dtype, width):
    table, w, eps = rnd(50, width, dtype=dtype), 1 + 0.3 * rnd(width, seed=1), 1e-3
    ids = torch.tensor([3, 0, 49, 3])
    e = table[ids].double()
    norm = lambda x: rms(x, eps) * w.double()
    x, xh = ops.embed_scaled(ids.to(DEV), table.to(DEV), 1.0, ops.padded(width), w.to(DEV), eps)
    assert torch.equal(x[:, :width].double().cpu(), e) and not x[:, width:].any() and not xh[:, width:].any() and xh.dtype == dtype
    tol = 2e-6 if dtype == torch.float32 else 6e-3
    close(xh[:, :width], norm(e), tol)
    before = rnd(4, width, seed=2)
    x[:, :width] = before.to(DEV)
    again, again_h = ops.embed_scaled(ids.to(DEV), table.to(DEV), 1.0, ops.padded(width), w.to(DEV), eps, add_to=(x, xh))
    assert again.data_ptr() == x.data_ptr() and again_h.data_ptr() == xh.data_ptr()
    close(x[:, :width], before.double() + e, 1e-6)
    close(xh[:, :width], norm(before.double() + e), tol)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [72, 101, 1536, 4096, 9000])
@pytest.mark.parametrize("mult", [1.0, 0.37])
def test_residual_between_two_norms(dtype, width, mult):
    T, eps, stride = 5, 1e-3, ops.padded(width)
    x = torch.zeros(T, stride)
    x[:, :width] = rnd(T, width, seed=1)
    y, w, nxt = (rnd(T, width, seed=2) * 0.05).to(dtype), rnd(width, seed=3), 1 + 0.3 * rnd(width, seed=4)
    want = x[:, :width].double() + mult * rms(y.double(), eps) * w.double()
    for next_norm in (nxt.to(DEV), None):
        xd, xh = x.to(DEV), torch.full((T, stride), 7.0, dtype=dtype, device=DEV)
        ops.residual_norm(xd, xh if next_norm is not None else None, y.to(DEV), w.to(DEV), eps, None, mult, next_norm)
        close(xd[:, :width], want, 1e-6)
        if next_norm is not None:
            close(xh[:, :width], rms(want, eps) * nxt.double(), 2e-6 if dtype == torch.float32 else 6e-3)
            assert (xh[:, width:] == 7.0).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,ff", [(1, 8), (3, 33), (70, 200), (300, 1024)])
def test_silu_gate(dtype, T, ff):
    both = rnd(T, 2 * ff, seed=1) * 4
    both[0, 0], both[-1, ff - 1] = -80.0, 80.0
    both = both.to(dtype)
    z, u = both[:, :ff].double(), both[:, ff:].double()
    close(ops.silu_gate(both.to(DEV), ff), z * torch.sigmoid(z) * u, 1e-6 if dtype == torch.float32 else 6e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,cap", [(1, 30.0), (7, 2.5), (1500, 30.0)])
def test_soft_cap(dtype, n, cap):
    x = (rnd(3, n, seed=2) * 2 * cap).to(dtype)
    x[0, 0] = 1e4
    out = ops.soft_cap(x.to(DEV), cap)
    assert out.dtype == torch.float32
    close(out, soft_cap(x.double(), cap), 1e-6)


@pytest.mark.parametrize("spec", [ops.RotarySpec(6, 50.0, 1.0), ops.RotarySpec(96, 1e6, 4.0), ops.RotarySpec(150, 1e4, 2.5)])
def test_rotary_table_far_away(spec):
    """Positions beyond what fp32 angles resolve, of sequences that stand at different places, and the table's reuse in a step."""
    cache = HybridCache([ops.WindowSpec(1, 1, 160, 8, 4, 0, 1.0)], torch.float32, DEV, 4)
    cache.allocate(4)
    past, lens, slots = [0, 131, 1000003, 7], [3, 70, 2, 1], [3, 1, 0, 2]
    for s, p in enumerate(past):
        cache.seen[s, 0] = p
    batch = cache.batch(lens, slots)
    freq = spec.frequencies().to(DEV)
    table = ops.rotary_table(spec, freq, batch)
    pos = torch.cat([past[s] + torch.arange(n, dtype=torch.float64) for s, n in zip(slots, lens)])
    ang = pos[:, None] * ref.rotation_frequencies(spec.dims, spec.base, spec.factor)[None]
    assert (table.double().cpu() - torch.cat([ang.cos(), ang.sin()], 1)).abs().max() < 2e-7
    assert ops.rotary_table(spec, freq, batch) is table


# ---- attention -----------------------------------------------------------------------------------------
class Layer:
    """One attention layer's sizes and random norm weights and biases, and what the oracle makes of projection rows."""

    def __init__(self, heads, kv_heads, dim, vdim, window, rot, scale, base=300.0, factor=2.0, sharp=False, keep=0):
        # sharp: constant norm weights, so that a direction survives the norm; a matching query scores 8, others about 8 / sqrt(dim)
        scale = 8.0 / (9.0 * dim) if sharp else scale
        self.spec = ops.WindowSpec(heads, kv_heads, dim, vdim, window, keep, scale, head_gate=True, sink=True)
        self.rot = ops.RotarySpec(rot, base, factor) if rot else None
        self.sizes = [heads * dim, kv_heads * dim, kv_heads * vdim, heads]
        self.offs = [0, self.sizes[0], sum(self.sizes[:2]), sum(self.sizes[:3])]
        self.cols = ops.padded(sum(self.sizes), 8)
        self.qw, self.kw = (torch.full((dim,), 3.0),) * 2 if sharp else (1 + 0.3 * rnd(dim, seed=11), 1 + 0.3 * rnd(dim, seed=12))
        self.bias = 0.5 * rnd(self.cols, seed=13)
        self.bias[self.offs[3]:] = 0.0
        self.eps = 1e-5

    def turn(self, x, first=0):
        return ref.rotate(x, first, self.rot.dims, self.rot.base, self.rot.factor) if self.rot else x

    def rows(self, n, seed):
        out = torch.zeros(n, self.cols)
        out[:, :sum(self.sizes)] = rnd(n, sum(self.sizes), seed=seed)
        return out

    def point(self, rows, qi, kj, sign=1.0):
        """The query at qi points exactly at the key at kj (or away from it), rotation included."""
        s, o = self.spec, self.offs
        u = rnd(s.kv_heads, s.dim, seed=1000 + kj)
        rows[kj, o[1]:o[2]] = 4 * u.reshape(-1) - self.bias[o[1]:o[2]]
        back = self.turn(u.double()[None], kj - qi)[0].float()                # turned on by qi, it meets the key turned by kj
        rows[qi, :o[1]] = 4 * sign * back.repeat_interleave(s.heads // s.kv_heads, 0).reshape(-1) - self.bias[:o[1]]

    def want(self, rows, dtype):
        s, o = self.spec, self.offs
        b = rows.double() + self.bias.double()
        q = self.turn(rms(b[:, :o[1]].reshape(-1, s.heads, s.dim), self.eps) * self.qw.double())
        k = self.turn(rms(b[:, o[1]:o[2]].reshape(-1, s.kv_heads, s.dim), self.eps) * self.kw.double())
        v = b[:, o[2]:o[3]].reshape(-1, s.kv_heads, s.vdim)
        if dtype == torch.bfloat16:
            q, k, v = (x.to(dtype).double() for x in (q, k, v))
        out = ref.sink_window_attention(q, k, v, s.scale, s.window) * torch.sigmoid(rows.double()[:, o[3]:o[3] + s.heads, None])
        return out.reshape(-1, s.heads * s.vdim)

    def step(self, proj, state, batch):
        if not hasattr(self, "dev"):
            self.dev = [t.to(DEV) for t in (self.qw, self.kw, self.bias)] + [self.rot.frequencies().to(DEV) if self.rot else None]
        qw, kw, bias, freq = self.dev
        table = ops.rotary_table(self.rot, freq, batch) if self.rot else None
        return ops.window_attention(proj, self.offs, qw, kw, self.eps, self.spec, state, batch, ops.HeadForm(bias, table))


def run(layer, dtype, seqs, cuts, edit=None, tol=None):
    """Rows of several sequences through the cache in portions (``cuts``: per sequence a list of portion lengths, all sequences
    advance together); everything is compared with the oracle.  ``edit(rows)`` changes the first sequence's rows."""
    rows = [layer.rows(n, 20 + i) for i, n in enumerate(seqs)]
    if edit:
        edit(rows[0])
    rows = [r.to(dtype) for r in rows]
    cache = HybridCache([layer.spec], dtype, DEV, num_slots=len(seqs) + 1)
    for t in cache.layers_state[0].values():
        t.fill_(float("nan") if dtype == torch.float32 else 7.0)              # whatever a slot held before must not matter
    slots = cache.allocate(len(seqs) + 1)[1:]
    got, at = [[] for _ in seqs], [0] * len(seqs)
    for step in range(max(len(c) for c in cuts)):
        live = [b for b in range(len(seqs)) if step < len(cuts[b])]
        lens = [cuts[b][step] for b in live]
        proj = torch.cat([rows[b][at[b]:at[b] + n] for b, n in zip(live, lens)]).to(DEV)
        batch = cache.batch(lens, [slots[b] for b in live])
        out = layer.step(proj, cache.layers_state[0], batch)
        cache.advance(batch)
        for b, part in zip(live, out.split(lens)):
            got[b].append(part)
            at[b] += part.shape[0]
    assert at == list(seqs)
    for b in range(len(seqs)):
        close(torch.cat(got[b]), layer.want(rows[b], dtype), tol or (5e-6 if dtype == torch.float32 else 1.5e-2), f"sequence {b} of {seqs}, cut {cuts[b][:4]}")


LAYERS = {
    "tiny": (3, 1, 8, 16, 5, 8, 0.5),
    "one_token_window": (2, 2, 64, 48, 1, 32, 0.125),
    "odd": (6, 2, 20, 36, 17, 10, 0.3),
    "odd_turn": (5, 5, 24, 8, 12, 22, 0.3),
    "no_turn": (4, 2, 32, 40, 33, 0, 0.2),
    "group_of_eight": (8, 1, 128, 128, 70, 128, 0.09),
    "group_of_twelve": (12, 1, 40, 8, 33, 16, 0.2),
    "between_tiles": (6, 2, 96, 72, 50, 64, 0.12),
    "between_tiles_values": (4, 1, 72, 88, 90, 32, 0.15),
    "wide": (4, 2, 200, 96, 64, 48, 0.07),
    "long_window": (4, 1, 64, 64, 300, 64, 0.15),
    "widest": (2, 1, 320, 272, 40, 320, 0.05),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(LAYERS))
def test_prompts_portions_and_decode(name, dtype):
    layer = Layer(*LAYERS[name])
    w = layer.spec.window
    seqs = [1, w + 1, 2 * w + 150, 65]
    run(layer, dtype, seqs, [[n] for n in seqs])                                           # whole prompts, unequal lengths
    run(layer, dtype, [7, w + 12], [[1] * 7, [1] * (w + 12)])                              # decoding from the first token on
    n = 2 * w + 40
    run(layer, dtype, [n, n], [[n - 20] + [1] * 20, [n - 20] + [1] * 20])
    for cut in sorted({2, 3, w, w + 1, 64, 65}):
        if n // cut < 120:
            run(layer, dtype, [n], [[cut] * (n // cut) + ([n % cut] if n % cut else [])])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["tiny", "odd", "group_of_eight", "long_window"])
@pytest.mark.parametrize("how", ["prompt", "decode", "portions"])
def test_one_key_stands_out(name, dtype, how):
    """A query points at one key: the oldest token inside the window, the one that has just left it, the token itself, and tokens
    at tile borders.  A window that is one token off, a wrong angle or a wrong row changes the output completely."""
    layer = Layer(*LAYERS[name], sharp=True)
    w = layer.spec.window
    n = 2 * w + 70
    qi = n - 3
    for kj in sorted(k for k in {qi - w + 1, qi - w + 2, qi - w, qi - w - 1, qi, qi - 1, 63, 64, 0} if 0 <= k <= qi):
        cuts = {"prompt": [n], "decode": [n - 6] + [1] * 6, "portions": [50] * ((n - 6) // 50) + [(n - 6) % 50 or 2] + ([6] if (n - 6) % 50 else [4])}[how]
        assert sum(cuts) == n
        run(layer, dtype, [n], [cuts], edit=lambda r: layer.point(r, qi, kj), tol=2e-5 if dtype == torch.float32 else 2.5e-2)


def test_sensitivity_of_the_edge_test():
    """The inputs above tell windows and positions apart."""
    layer = Layer(*LAYERS["odd"], sharp=True)
    s, w, qi = layer.spec, layer.spec.window, 40
    rows = layer.rows(44, 5)
    layer.point(rows, qi, qi - w + 1)
    base = layer.want(rows, torch.float32)[qi]
    layer.spec = ops.WindowSpec(s.heads, s.kv_heads, s.dim, s.vdim, w - 1, 0, s.scale, True, True)
    assert (layer.want(rows, torch.float32)[qi] - base).abs().max() > 0.3
    layer.spec, layer.rot = s, ops.RotarySpec(layer.rot.dims, layer.rot.base, 1.0)
    assert (layer.want(rows, torch.float32)[qi] - base).abs().max() > 0.1


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("how", ["prompt", "decode"])
@pytest.mark.parametrize("name", ["tiny", "no_turn", "group_of_eight", "long_window"])
def test_sink_takes_most_of_the_weight(name, dtype, how):
    """Scores far below 0, so that the sink holds nearly all, half, or far more than fp32 resolves; scores far above leave it nothing."""
    args = list(LAYERS[name])
    args[4] = 3 if args[4] < 100 else args[4]
    layer = Layer(*args, sharp=True)
    s, n = layer.spec, 130
    shape = [n] if how == "prompt" else [1] * n

    def aim(strength):
        """One direction for every key; queries along it, in units of the resulting score before rotation."""
        def edit(rows):
            o = layer.offs
            u = torch.sign(rnd(s.kv_heads, s.dim, seed=77))
            for t in range(n):
                layer.point(rows, t, t)
                rows[t, o[1]:o[2]] = u.reshape(-1) - layer.bias[o[1]:o[2]]
                rows[t, :o[1]] = (1.0 if strength > 0 else -1.0) * u.repeat_interleave(s.heads // s.kv_heads, 0).reshape(-1) - layer.bias[:o[1]]
        return edit
    for target in (-3.0, -0.7, 0.7, 60.0, -60.0, -400.0):
        layer.spec = ops.WindowSpec(s.heads, s.kv_heads, s.dim, s.vdim, s.window, 0, abs(target) / (9.0 * s.dim), True, True)
        if target <= -60.0:
            # nothing is left but the sink: the outputs vanish, whatever the tolerance relative to them
            rows = layer.rows(n, 20)
            aim(target)(rows)
            cache = HybridCache([layer.spec], dtype, DEV, num_slots=1)
            cache.allocate(1)
            out, at = [], 0
            for c in shape:
                batch = cache.batch([c])
                out.append(layer.step(rows[at:at + c].to(dtype).to(DEV), cache.layers_state[0], batch))
                cache.advance(batch)
                at += c
            out, want = torch.cat(out).double().cpu(), layer.want(rows.to(dtype), dtype)
            assert torch.isfinite(out).all() and (out - want).abs().max() < (1e-3 if dtype == torch.float32 else 0.1) * rows.abs().max() and out[0].abs().max() < 1e-8
        else:
            run(layer, dtype, [n], [shape], edit=aim(target), tol=2e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_biases_norms_and_rotation_may_each_be_absent(dtype):
    H, G, D, Dv, T = 4, 2, 32, 24, 9
    proj = rnd(T, (H + G) * D + G * Dv + 8, seed=3).to(dtype)
    spec = ops.WindowSpec(H, G, D, Dv, 4, 0, 0.3, head_gate=True, sink=False)
    offs = [0, H * D, (H + G) * D, (H + G) * D + G * Dv]
    for bias, norm in ((None, None), (0.4 * rnd(proj.shape[1], seed=4), None), (None, 1 + 0.2 * rnd(D, seed=5))):
        cache = HybridCache([spec], dtype, DEV, 1)
        cache.allocate(1)
        batch = cache.batch([T])
        got = ops.window_attention(proj.to(DEV), offs, None if norm is None else norm.to(DEV), None if norm is None else norm.to(DEV), 1e-5, spec, cache.layers_state[0], batch,
                                   ops.HeadForm(None if bias is None else bias.to(DEV), None))
        b = proj.double() + (0 if bias is None else bias.double())
        form = lambda x: x if norm is None else rms(x, 1e-5) * norm.double()
        q, k, v = form(b[:, :offs[1]].reshape(T, H, D)), form(b[:, offs[1]:offs[2]].reshape(T, G, D)), b[:, offs[2]:offs[3]].reshape(T, G, Dv)
        if dtype == torch.bfloat16:
            q, k, v = (x.to(dtype).double() for x in (q, k, v))
        age = torch.arange(T)[:, None] - torch.arange(T)[None]
        want = torch.stack([torch.softmax(((q[:, h] @ k[:, h // 2].T) * 0.3).masked_fill((age < 0) | (age >= 4), -float("inf")), -1) @ v[:, h // 2] for h in range(H)], 1)
        want = (want * torch.sigmoid(proj.double()[:, offs[3]:offs[3] + H, None])).reshape(T, H * Dv)
        close(got, want, 5e-6 if dtype == torch.float32 else 1.5e-2)
