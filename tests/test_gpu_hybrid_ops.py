"""The mechanisms of the hybrid decoders one by one against the plain oracle (oracle/hybrid_ref.py), on the GPU."""
import pytest
import torch

from oracle import hybrid_ref as ref
from trimkv_amd import hybrid_ops as ops
from trimkv_amd.hybrid_cache import HybridCache

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]


def close(got, want, tol, what=""):
    got = got.detach().double().cpu()
    err = (got - want).abs().max().item() / max(want.abs().max().item(), 1e-30)
    assert err <= tol, f"{what}: error {err:.3e} of the largest value, tolerance {tol:.1e}"


def rnd(*shape, seed=0, dtype=torch.float32):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)).to(dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [40, 100, 192])
def test_embedding_scale_and_padding(dtype, width):
    table = rnd(50, width, dtype=dtype)
    ids = torch.tensor([3, 0, 49, 3])
    x, xh = ops.embed_scaled(ids.to(DEV), table.to(DEV), 2.75, ops.padded(width))
    close(x[:, :width], table[ids].double() * 2.75, 1e-7)
    assert not x[:, width:].any()
    if dtype == torch.bfloat16:
        assert torch.equal(xh, x.to(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,n,k", [(1, 3, 64), (17, 40, 352), (70, 16, 1024), (2100, 33, 192), (2050, 130, 128)])
def test_linear_keeps_fp32(dtype, rows, n, k):
    x, w = rnd(rows, k, seed=1) * 3.0, rnd(n, k, seed=2, dtype=dtype)
    out = ops.linear_f32(x.to(DEV), w.to(DEV))
    close(out, x.double() @ w.double().T, 2e-6)        # the fp32 input is not rounded to the weights' 16 bits on the way


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,top", [(72, 1), (101, 3), (1536, 1), (4096, 8)])
def test_residual_norm(dtype, width, top):
    T, eps, stride = 5, 1e-3, ops.padded(width)
    x = torch.zeros(T, stride)
    x[:, :width] = rnd(T, width, seed=1)
    y, w = (rnd(T * top, width, seed=2) * 0.05).to(dtype), rnd(width, seed=3)
    wt = torch.rand(T, top, generator=torch.Generator().manual_seed(4)) if top > 1 else None
    summed = y.double().view(T, top, width) * (1.0 if wt is None else wt.double()[:, :, None])
    want = x[:, :width].double() + ref.rms(summed.sum(1), eps) * w.double()
    xd = x.to(DEV)
    xh = torch.empty(T, stride, dtype=dtype, device=DEV) if dtype != torch.float32 else None
    ops.residual_norm(xd, xh, y.to(DEV), w.to(DEV), eps, None if wt is None else wt.to(DEV))
    close(xd[:, :width], want, 1e-6)
    if xh is not None:
        assert torch.equal(xh[:, :width], xd[:, :width].to(dtype))
    rows = torch.tensor([4, 0, 4])
    out = ops.rms_rows(xd, rows.to(DEV), w.to(DEV), eps, dtype)
    close(out, (ref.rms(want, eps) * w.double())[rows], 1e-6 if dtype == torch.float32 else 6e-3)


# ---- windowed attention ------------------------------------------------------------------------------
def run_window(spec, dtype, seqs, cuts, stand_out=()):
    """Projection rows of several sequences through the cache in portions (``cuts``: per sequence a list of portion lengths,
    all sequences advance together); compares everything with the oracle.  ``stand_out``: (sequence, query position, key
    position) whose q and k are made to point the same way, far above all other scores."""
    s, eps = spec, 1e-5
    H, G, D, Dv = s.heads, s.kv_heads, s.dim, s.vdim
    qw, kw = 1 + 0.3 * rnd(H * D, seed=11), 1 + 0.3 * rnd(G * D, seed=12)
    sizes = [H * D, G * D, G * Dv, H * Dv]
    offs = [0, sizes[0], sizes[0] + sizes[1], sum(sizes[:3])]
    rows = [rnd(n, sum(sizes), seed=20 + i) for i, n in enumerate(seqs)]
    for b, qi, kj in stand_out:
        u = rnd(G, D, seed=1000 + kj) * 6.0          # one direction per KV head, shared by its query heads
        rows[b][kj, offs[1]:offs[2]] = u.reshape(-1)
        rows[b][qi, :offs[1]] = u.repeat_interleave(H // G, dim=0).reshape(-1)
    rows = [r.to(dtype) for r in rows]
    want = []
    for r in rows:
        r = r.double()
        q = (ref.rms(r[:, :offs[1]], eps) * qw.double()).view(-1, H, D)
        k = (ref.rms(r[:, offs[1]:offs[2]], eps) * kw.double()).view(-1, G, D)
        if dtype == torch.bfloat16:
            q, k = q.to(dtype).double(), k.to(dtype).double()
        o = ref.window_attention(q, k, r[:, offs[2]:offs[3]].reshape(-1, G, Dv), s.scale, s.window, s.keep_first)
        want.append(o.reshape(-1, H * Dv) * torch.sigmoid(r[:, offs[3]:]))
    cache = HybridCache([spec], dtype, DEV, num_slots=len(seqs) + 1)
    for t in cache.layers_state[0].values():
        t.fill_(float("nan") if dtype == torch.float32 else 7.0)          # whatever a slot held before must not matter
    slots = cache.allocate(len(seqs) + 1)[1:]
    got = [[] for _ in seqs]
    at = [0] * len(seqs)
    for step in range(max(len(c) for c in cuts)):
        live = [b for b in range(len(seqs)) if step < len(cuts[b])]
        lens = [cuts[b][step] for b in live]
        proj = torch.cat([rows[b][at[b]:at[b] + n] for b, n in zip(live, lens)]).to(DEV)
        batch = cache.batch(lens, [slots[b] for b in live])
        out = ops.window_attention(proj, offs, qw.to(DEV), kw.to(DEV), eps, s, cache.layers_state[0], batch)
        cache.advance(batch)
        for b, part in zip(live, out.split(lens)):
            got[b].append(part)
            at[b] += part.shape[0]
    for b, n in enumerate(seqs):
        assert at[b] == n
        close(torch.cat(got[b]), want[b], 3e-6 if dtype == torch.float32 else 1.2e-2, f"sequence {b} of {seqs}, cut {cuts[b][:4]}")


SPECS = {
    "tiny": ops.WindowSpec(3, 1, 8, 16, 5, 2, 0.4),
    "odd": ops.WindowSpec(6, 2, 20, 36, 17, 0, 0.3),
    "one_head_each": ops.WindowSpec(2, 2, 64, 48, 1, 1, 0.125),
    "group_of_eight": ops.WindowSpec(8, 1, 128, 128, 70, 64, 0.09),
    "group_of_twelve": ops.WindowSpec(12, 1, 40, 8, 33, 65, 0.2),
    "wide": ops.WindowSpec(4, 2, 200, 96, 64, 4, 0.07),
    "long_window": ops.WindowSpec(4, 1, 64, 64, 300, 30, 0.15),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(SPECS))
def test_window_prompts_and_decode(name, dtype):
    s = SPECS[name]
    edge = s.keep_first + s.window
    seqs = [1, edge + 1, 2 * edge + 150, 65]
    run_window(s, dtype, seqs, [[n] for n in seqs])                                        # whole prompts, unequal lengths
    run_window(s, dtype, [7, edge + 12], [[1] * 7, [1] * (edge + 12)])                     # decoding from the first token on
    n = 2 * edge + 40
    run_window(s, dtype, [n, n], [[n - 20] + [1] * 20, [n - 20] + [1] * 20])
    for cut in (2, 3, s.window, edge, 64, 65):
        if n // cut < 120:
            run_window(s, dtype, [n], [[cut] * (n // cut) + ([n % cut] if n % cut else [])])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["tiny", "group_of_eight", "group_of_twelve", "long_window"])
@pytest.mark.parametrize("how", ["prompt", "decode", "portions"])
def test_window_edges_stand_out(name, dtype, how):
    """One query points at one key: the last kept token and the first not kept, the oldest token inside the window and the one
    that has just left it.  A window or a kept prefix that is one token off changes the output completely."""
    s = SPECS[name]
    n = 2 * (s.window + s.keep_first) + 70
    qi = n - 3
    keys = [max(s.keep_first - 1, 0), s.keep_first, qi - s.window + 1, qi - s.window, qi - s.window - 1, qi, 0, 63, 64]
    for kj in sorted(set(k for k in keys if 0 <= k <= qi)):
        cuts = {"prompt": [n], "decode": [n - 6] + [1] * 6, "portions": [50] * ((n - 6) // 50) + [(n - 6) % 50 or 2] + ([6] if (n - 6) % 50 else [4])}[how]
        assert sum(cuts) == n
        run_window(s, dtype, [n], [cuts], stand_out=[(0, qi, kj)])


def test_window_sensitivity_of_the_edge_test():
    """The inputs of the edge test tell windows apart: with the key just inside, a window one token shorter moves the output."""
    s = SPECS["tiny"]
    u = rnd(1, 8, seed=5) * 6
    q, k, v = rnd(30, 3, 8, seed=6), rnd(30, 1, 8, seed=7), rnd(30, 1, 16, seed=8)
    k[24 - s.window + 1] = u
    q[24] = u.repeat(3, 1)
    a, b = (ref.window_attention(q, k, v, s.scale, w, s.keep_first)[24] for w in (s.window, s.window - 1))
    assert (a - b).abs().max() > 0.5


# ---- mLSTM ---------------------------------------------------------------------------------------------
def run_mlstm(spec, dtype, seqs, cuts, gate_scale=1.0, f_shift=2.0, tol=None):
    s, eps = spec, 1e-5
    H, D, Dv = s.heads, s.dim, s.vdim
    sizes = [H * D, H * D, H * Dv, H * Dv]
    offs = [0, sizes[0], 2 * sizes[0], sum(sizes[:3])]
    rows = [rnd(n, sum(sizes), seed=30 + i).to(dtype) for i, n in enumerate(seqs)]
    raw = [rnd(n, 2 * H, seed=60 + i) * gate_scale for i, n in enumerate(seqs)]
    ib, fb, w = rnd(H, seed=90), f_shift + rnd(H, seed=91), 1 + 0.3 * rnd(H * Dv, seed=92)
    want = []
    for r, z in zip(rows, raw):
        r, z = r.double(), z.double()
        li = ref.soft_cap(z[:, :H] + ib.double(), s.gate_cap)
        lf = torch.nn.functional.logsigmoid(ref.soft_cap(z[:, H:] + fb.double(), s.gate_cap))
        o, _ = ref.mlstm_scan(r[:, :offs[1]].reshape(-1, H, D) * D ** -0.5, r[:, offs[1]:offs[2]].reshape(-1, H, D), r[:, offs[2]:offs[3]].reshape(-1, H, Dv), li, lf)
        want.append(ref.rms(o, eps).reshape(-1, H * Dv) * w.double() * torch.sigmoid(r[:, offs[3]:]))
    cache = HybridCache([spec], dtype, DEV, num_slots=len(seqs) + 1)
    for t in cache.layers_state[0].values():
        t.fill_(float("nan"))                                   # a fresh sequence starts from zero whatever the slot held
    slots = cache.allocate(len(seqs) + 1)[1:]
    got, at = [[] for _ in seqs], [0] * len(seqs)
    for step in range(max(len(c) for c in cuts)):
        live = [b for b in range(len(seqs)) if step < len(cuts[b])]
        lens = [cuts[b][step] for b in live]
        proj = torch.cat([rows[b][at[b]:at[b] + n] for b, n in zip(live, lens)]).to(DEV)
        gates = torch.cat([raw[b][at[b]:at[b] + n] for b, n in zip(live, lens)]).to(DEV)
        batch = cache.batch(lens, [slots[b] for b in live])
        out = ops.mlstm(proj, offs, gates, ib.to(DEV), fb.to(DEV), w.to(DEV), eps, s, cache.layers_state[0], batch)
        cache.advance(batch)
        for b, part in zip(live, out.split(lens)):
            got[b].append(part)
            at[b] += part.shape[0]
    for b, n in enumerate(seqs):
        assert at[b] == n
        close(torch.cat(got[b]), want[b], tol or (2e-5 if dtype == torch.float32 else 1e-2), f"sequence {b} of {seqs}, cut {cuts[b][:4]}")


MSPECS = {
    "tiny": ops.MlstmSpec(2, 8, 16, 5.0),
    "odd": ops.MlstmSpec(3, 20, 36, 3.0),
    "mid": ops.MlstmSpec(2, 48, 72, 9.0),
    "wide_values": ops.MlstmSpec(1, 64, 200, 12.0),
    "square": ops.MlstmSpec(2, 128, 128, 15.0),
    "large": ops.MlstmSpec(1, 256, 136, 15.0),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MSPECS))
def test_mlstm_prompts_portions_and_decode(name, dtype):
    s = MSPECS[name]
    run_mlstm(s, dtype, [1, 64, 65, 200], [[1], [64], [65], [200]])
    run_mlstm(s, dtype, [90, 90], [[70] + [1] * 20] * 2)
    run_mlstm(s, dtype, [40], [[1] * 40])
    for cut in (2, 3, 63, 64, 65):
        run_mlstm(s, dtype, [140, 131], [[cut] * (140 // cut) + ([140 % cut] if 140 % cut else []), [cut] * (131 // cut) + ([131 % cut] if 131 % cut else [])])


@pytest.mark.parametrize("dtype", DTYPES)
def test_mlstm_segments_side_by_side(dtype):
    """Long prompts are cut into segments that run in parallel: segment borders, a sequence that ends inside the first one, a
    state from earlier portions, and decoding behind it."""
    s = ops.MlstmSpec(2, 32, 24, 8.0)
    run_mlstm(s, dtype, [1100, 70, 513], [[1100], [70], [513]], f_shift=5.0)
    run_mlstm(s, dtype, [1400], [[30, 1300] + [1] * 70], f_shift=6.0)
    run_mlstm(s, dtype, [1100], [[512, 580, 8]], f_shift=6.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("gate_scale,f_shift", [(30.0, 0.0), (1.0, 12.0), (1.0, -12.0)])
def test_mlstm_extreme_gates(dtype, gate_scale, f_shift):
    """Gates at their caps in both directions, nothing forgotten, everything forgotten: the running maximum carries it."""
    s = ops.MlstmSpec(2, 32, 48, 10.0)
    run_mlstm(s, dtype, [330], [[300] + [1] * 30], gate_scale, f_shift, tol=1e-4 if dtype == torch.float32 else 1e-2)


# ---- routed experts --------------------------------------------------------------------------------------
@pytest.mark.parametrize("E,top,count,keep", [(14, 3, 2, 1), (8, 2, 1, 1), (6, 2, 6, 2), (64, 8, 8, 4), (130, 7, 10, 3), (4, 4, 2, 2), (5, 1, 1, 1)])
def test_router(E, top, count, keep):
    z = rnd(300, E, seed=E) * 2
    for shift in (0.0, -3.0):              # all choice scores negative: a closed group must not win with a zero
        corr = 0.5 * rnd(E, seed=E + 1) + shift
        ids, wt = ops.route(z.to(DEV), corr.to(DEV), ops.RouterSpec(E, top, count, keep))
        want_ids, want_w = ref.choose_experts(z.double(), corr.double(), top, count, keep)
        assert torch.equal(ids.cpu().long(), want_ids)
        close(wt, want_w, 1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,E,top,ff,width", [(1, 6, 2, 40, 72), (5, 3, 1, 64, 64), (37, 10, 3, 24, 100), (700, 8, 3, 136, 200), (130, 4, 4, 320, 256), (900, 5, 2, 64, 520)])
def test_experts(dtype, T, E, top, ff, width):
    wp, fp = ops.padded(width), ops.padded(ff)
    x = torch.zeros(T, wp)
    x[:, :width] = rnd(T, width, seed=1)
    up, down = torch.zeros(E, fp, wp), torch.zeros(E, wp, fp)
    up[:, :ff, :width] = rnd(E, ff, width, seed=2) * width ** -0.5
    down[:, :width, :ff] = rnd(E, width, ff, seed=3) * ff ** -0.5
    x, up, down = x.to(dtype), up.to(dtype), down.to(dtype)
    gen = torch.Generator().manual_seed(4)
    ids = torch.stack([torch.randperm(E, generator=gen)[:top] for _ in range(T)]).int()
    if E > 4:
        ids[ids == 2] = 0 if top == 1 else ids[ids == 2]          # an expert nobody asks for
    y = ops.experts(x.to(DEV), ids.to(DEV), ops.pack_matrix(up).contiguous().to(DEV), ops.pack_matrix(down).contiguous().to(DEV), width).view(T, top, width)
    want = torch.stack([torch.stack([ref.expert(x[t].double()[:width], up[e].double()[:ff, :width], down[e].double()[:width, :ff]) for e in ids[t].tolist()]) for t in range(T)])
    close(y, want, 2e-6 if dtype == torch.float32 else 1.2e-2)
