"""Siterax end to end on the GPU against the plain oracle: the stream behind every layer, prompts, portions, decoding, unequal
batches, slots that are used again, greedy generation (eager and replayed), loading from disk, trace replay."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

from trimkv_amd import registry
from trimkv_amd.graphed import GraphedDecoder
from tests.hybrid_util import DEV, assert_rows, row_error, tokens
from tests.siterax_util import CONFIGS, build, oracle, weights
from tests.test_gpu_hybrid_model import packed_step

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
_cache = {}


def case(name, n, seed=1):
    """Configuration, weights, tokens and the oracle's logits (kept: several tests share them)."""
    cfg = CONFIGS[name]
    if name not in _cache:
        _cache[name] = weights(cfg)
    key = (name, n, seed)
    if key not in _cache:
        toks = tokens(cfg, n, seed)
        _cache[key] = (toks, oracle(cfg, _cache[name], toks))
    return (cfg, _cache[name], *_cache[key])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_stream_behind_every_layer(name, dtype):
    cfg, w, toks, want = case(name, 60)
    model = build(cfg, w, dtype)
    layers, ours = [], []
    oracle(cfg, w, toks, layers_out=layers)
    out = model(torch.tensor([toks], device=DEV), layers_out=ours)
    assert len(layers) == len(ours)
    for n, (a, b) in enumerate(zip(ours, layers)):
        assert float(row_error(a, b).max()) < (1e-5 if dtype == torch.float32 else 0.05), f"layer run {n}"
    assert_rows(out.logits[0], want, dtype)
    assert float(out.logits.abs().max()) <= cfg["logit_softcap"]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_portions_and_decode(name, dtype):
    cfg, w, toks, want = case(name, 190)
    model = build(cfg, w, dtype)
    whole = model(torch.tensor([toks], device=DEV)).logits[0]
    assert_rows(whole, want, dtype, "whole prompt")
    for cuts in ([2] * 10 + [170], [64, 65, 1, 60], [1] * 40 + [150], [120] + [1] * 70):
        cache, rows, at = model.new_cache(), [], 0
        (slot,) = cache.allocate(1)
        for n in cuts:
            rows.append(packed_step(model, cache, [toks[at:at + n]], [slot])[0])
            at += n
        assert_rows(torch.cat(rows), want, dtype, f"cut {cuts[:3]}")
        # beyond rounding, the cut must not matter
        assert float(row_error(torch.cat(rows), whole.double().cpu()).max()) < (2e-5 if dtype == torch.float32 else 0.06)
        assert cache.get_seq_length() == 190 and cache.seen[slot].tolist() == [190, len(cuts)]


@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_batches_and_slots_used_again(dtype):
    lens = (1 + 12, 40 + 5, 23 + 30, 97 + 30, 9 + 11)
    cfg, w = CONFIGS["looped_middle"], case("looped_middle", 60)[1]
    model = build(cfg, w, dtype)
    cache = model.new_cache(2)
    seqs, want = zip(*(case("looped_middle", n, seed=10 + i)[2:] for i, n in enumerate(lens)))
    rows = [[] for _ in seqs]

    def run(ids, counts, slots):
        parts = []
        for i, n in zip(ids, counts):
            at = sum(r.shape[0] for r in rows[i])
            parts.append(seqs[i][at:at + n])
        for i, r in zip(ids, packed_step(model, cache, parts, [slots[i] for i in ids])):
            rows[i].append(r)

    slots = {i: cache.allocate(1)[0] for i in range(4)}            # grows past the two slots it was made with
    run([0, 1, 2, 3], [1, 40, 23, 97], slots)
    for _ in range(5):
        run([3, 1, 0, 2], [1] * 4, slots)                           # another order of the same batch
    cache.release([slots[1]])
    for _ in range(7):
        run([0, 2, 3], [1] * 3, slots)
    cache.release([slots[0]])
    slots[4] = cache.allocate(1)[0]
    run([4, 2], [9, 1], slots)                                      # a prompt beside a decoding sequence
    for _ in range(11):
        run([2, 4, 3], [1] * 3, slots)
    for _ in range(6):
        run([3, 2], [1] * 2, slots)
    run([3], [1], slots)
    for i in range(5):
        assert_rows(torch.cat(rows[i]), want[i], dtype, f"sequence {i}")


def test_every_slot_is_used_again_and_again():
    cfg, w = CONFIGS["looped_to_the_end"], case("looped_to_the_end", 60)[1]
    model = build(cfg, w, torch.float32)
    cache = model.new_cache(2)
    for turn in range(4):
        slots = cache.allocate(2)
        a, wa = case("looped_to_the_end", 100 - 30 * turn + 10, 50 + turn)[2:]
        b, wb = case("looped_to_the_end", 17, 60 + turn)[2:]
        n = len(a) - 10
        first = packed_step(model, cache, [a[:n], b[:7]], slots)
        rest = [packed_step(model, cache, [[a[n + k]], [b[7 + k]]], slots) for k in range(10)]
        assert_rows(torch.cat([first[0]] + [r[0] for r in rest]), wa, torch.float32, f"turn {turn}")
        assert_rows(torch.cat([first[1]] + [r[1] for r in rest]), wb, torch.float32, f"turn {turn}")
        cache.release(slots)
    assert cache.num_slots == 2


@pytest.mark.parametrize("name", ["looped_middle", "one_layer_often"])
def test_long_decode(name):
    cfg, w, toks, want = case(name, 420, 7)
    model = build(cfg, w, torch.float32)
    cache = model.new_cache()
    slot = cache.allocate(1)
    rows = [packed_step(model, cache, [toks[:20]], slot)[0]] + [packed_step(model, cache, [[t]], slot)[0] for t in toks[20:]]
    assert_rows(torch.cat(rows), want, torch.float32)


def greedy(cfg, w, prompt, n):
    out, margins = list(prompt), []
    for _ in range(n):
        two = oracle(cfg, w, out)[-1].topk(2)
        margins.append(float(two.values[0] - two.values[1]))
        out.append(int(two.indices[0]))
    assert min(margins) > 1e-3, "choose another seed: the oracle's choice is too close"
    return out


def test_generate():
    cfg, w = CONFIGS["looped_middle"], case("looped_middle", 60)[1]
    model = build(cfg, w, torch.float32)
    prompts = [tokens(cfg, 26, 70), tokens(cfg, 26, 71)]
    wanted = [greedy(cfg, w, p, 14) for p in prompts]
    uneq = [tokens(cfg, n, 80 + n) for n in (3, 31, 12)]
    ids = torch.zeros(3, 31, dtype=torch.int64, device=DEV)
    for b, p in enumerate(uneq):
        ids[b, :len(p)] = torch.tensor(p, device=DEV)
    uneq_wanted = [greedy(cfg, w, p, 9) for p in uneq]
    for use_graph in (False, True):
        for chunk in (0, 2, 13):
            assert model.generate(torch.tensor(prompts, device=DEV), 14, prefill_chunk=chunk, use_graph=use_graph).tolist() == wanted
            # unequal prompts, padded on the right: each as alone
            together = model.generate(ids, 9, prefill_chunk=chunk, use_graph=use_graph, lengths=[len(p) for p in uneq])
            assert [g.tolist() for g in together] == uneq_wanted


@pytest.mark.parametrize("dtype", DTYPES)
def test_replayed_steps_equal_eager_ones(dtype):
    """Several replays with eager work on another cache between them; sequences that end make the step be captured anew."""
    cfg, w = CONFIGS["looped_middle"], case("looped_middle", 60)[1]
    model = build(cfg, w, dtype)
    seqs = [tokens(cfg, 40, 90 + b) for b in range(3)]
    eager, replayed = model.new_cache(3), model.new_cache(3)
    for cache in (eager, replayed):
        cache.allocate(3)
        packed_step(model, cache, [s[:10 + b] for b, s in enumerate(seqs)], cache.active)
    dec = GraphedDecoder(model, replayed, logits_to_keep=1)
    for k in range(20):
        if k == 12:
            for cache in (eager, replayed):
                cache.release([cache.active[1]])
            seqs.pop(1)
            dec.close()
            dec = GraphedDecoder(model, replayed, logits_to_keep=1)
        ids = torch.tensor([[s[20 + k]] for s in seqs], device=DEV)
        a = model(ids, past_key_values=eager, logits_to_keep=1).logits
        torch.cuda.synchronize()
        b = dec(input_ids=ids).logits
        assert torch.equal(a, b), k
    dec.close()
    assert replayed.tokens_seen == eager.tokens_seen and torch.equal(replayed.seen, eager.seen)


def test_from_disk_and_trace_replay(tmp_path):
    """config.json + safetensors -> registry -> logits, and the same requests through bin/trace_run."""
    cfg, w, a, wa = case("looped_to_the_end", 30, 120)
    b, wb = case("looped_to_the_end", 12, 121)[2:]
    (tmp_path / "m").mkdir()
    (tmp_path / "out").mkdir()
    (tmp_path / "m" / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "m" / "model.safetensors"))
    model = registry.from_pretrained(str(tmp_path / "m"), torch_dtype=torch.float32).to(DEV)
    assert_rows(model(torch.tensor([a], device=DEV)).logits[0], wa, torch.float32)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:25], "want": [0, 24]}, {"id": "y", "tokens": b[:11], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": b[11:], "want": [0]}, {"id": "x", "tokens": a[25:26], "want": [0]}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": a[26:27], "want": []}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "z", "tokens": b, "want": list(range(12))}], "end": ["z"]}]
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", "float32", "--out", str(tmp_path / "out"),
                           "--max-tokens", "64"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    read = lambda i: torch.from_numpy(np.fromfile(tmp_path / "out" / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"]))
    assert_rows(read(0), wa[[0, 24]], torch.float32)
    assert_rows(read(1), torch.stack([wb[11], wa[25]]), torch.float32)
    assert not (tmp_path / "out" / "2.f32").exists()
    assert_rows(read(3), wb, torch.float32)
