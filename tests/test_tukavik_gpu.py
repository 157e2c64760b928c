"""Tukavik on the GPU against the plain implementation (tests/plain/tukavik_plain.py): the kernels of each new
mechanism alone (the step between two sublayers in all its modes, the recurrence over unequal requests in several
steps, position vectors, the product with xIELU behind it in every kernel that serves it, the pass behind queries
without a latent), one-layer models of each mixer and of the feed-forward, whole prompts against token-by-token
decoding and portions down to two tokens, mixed batches against each request alone with pages and slots that are freed
and used again, single keys far away and at page borders (with controls that a lost one moves the plain logits by many
times the bound), a far token that only the recurrence's state still holds, the first tokens, long decoding
through replayed graphs, generation through the scheduler, and the trace replay program."""

from __future__ import annotations

import json
import math
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

from helpers import feed, make_mixed_trace, max_live_tokens, random_tokens, rel_err, replay_in_process
from plain import tukavik_plain as plain
from tukavik_cases import CASES, SINGLE, bare, config, dense, latent, make_tensors, recurrence, write_model

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent

# Bounds on max |engine - plain| / max |plain logit| over a request, some three times the largest error
# measured on the MI355X on these weights.
TOL = {"float32": 4e-6, "bfloat16": 1.5e-2}
# (case C's recurrence of one channel feeds a layer norm with a small eps: where that one number is near zero, its
# rounding is multiplied by up to a thousand, on the whole row)
TOL_C = {"float32": 2e-5, "bfloat16": 5.5e-2}


def tol(dtype, name=""):
    return (TOL_C if name == "C" else TOL)[dtype]


def K():
    from lockstep_amd.ops import kernels
    return kernels()


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """(case, dtype) -> (loaded model, plain model, raw config, page size, folder), made once."""
    made = {}

    def get(name, dtype="float32", table=CASES, seed=11):
        from lockstep_amd import load_model

        key = (name, dtype, seed)
        if key not in made:
            case = table[name]
            tensors = make_tensors(case["raw"], seed=seed)
            folder = write_model(tmp_path_factory.mktemp(f"tukavik{name}"), case["raw"], tensors)
            made[key] = (load_model(folder, dtype=dtype), plain.PlainTukavik(case["raw"], tensors), case["raw"],
                         case["page_size"], folder)
        return made[key]

    return get


def new_cache(model, page_size, tokens=512, requests=4, poison=True):
    return model.make_cache(num_pages=-(-tokens // page_size), page_size=page_size, max_requests=requests,
                            max_tokens_per_request=tokens, poison_on_free=poison)


def step_meta(lengths, starts, slots):
    """tok_seq, tok_pos, seqs [n * 8] as the engine's upload lays them out."""
    seqs, tok_seq, tok_pos, off = [], [], [], 0
    for i, (n, s, slot) in enumerate(zip(lengths, starts, slots)):
        seqs.append([off, n, s, s + n, slot, 0, 0, 0])
        tok_seq += [i] * n
        tok_pos += list(range(s, s + n))
        off += n
    as_dev = lambda x: torch.tensor(x, dtype=torch.int32, device="cuda")  # noqa: E731
    return as_dev(tok_seq), as_dev(tok_pos), as_dev(seqs).reshape(-1)


def close(got, want, dtype, scale=1.0):
    tol = 1e-5 if dtype == torch.float32 else 1.6e-2
    return float((got.double().cpu() - want).abs().max()) <= tol * max(scale, float(want.abs().max()))


# ---------------------------------------------------------------------------
# the kernels of each mechanism alone
# ---------------------------------------------------------------------------

def plain_norm(x, norm):
    weight, eps, centred = norm
    f = plain.layer_norm if centred else plain.rms_norm
    return f(x, weight.double().cpu(), eps)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [3, 45, 64, 1000, 1536, 2500, 5000, 9001])
@pytest.mark.parametrize("centred", [True, False])
def test_the_step_between_two_sublayers(dtype, width, centred):
    """Addition, addition of a normed output, kept results, averages over one to eleven of them, the next norm; with
    rows far from zero, and with a row list that leaves the stream alone."""
    g = torch.Generator().manual_seed(width)
    t, layers = 5, 11
    draw = lambda *shape: torch.randn(shape, generator=g)  # noqa: E731
    norm = ((1 + 0.3 * draw(width)).cuda(), 1e-3, centred)
    post = ((1 + 0.3 * draw(width)).cuda(), 1e-5, not centred if width == 64 else centred)
    k = K()
    for slices, keep, averaged, with_post in ((0, 0, False, False), (1, 1, True, True), (3, 4, True, True), (11, 11, True, False),
                                              (9, 2, False, True), (2, 0, True, True)):
        h = draw(t, width) * 2 + 5
        parts = draw(slices, t, width) + 1 if slices else None
        results = draw(layers + 1, t, width)
        shares = draw(keep + 1)
        x = h.double()
        if slices:
            y = parts.double().sum(0)
            x = x + (plain_norm(y, post) if with_post else y)
        kept = results.double()
        kept[keep] = x
        if averaged:
            x = plain.depth_average(list(kept[:keep + 1]), shares.double())
        want = plain_norm(x, norm)
        dev, dres = h.cuda(), results.cuda()
        out = torch.empty((t, width), dtype=dtype, device="cuda")
        args = (parts.cuda() if slices else None, post if with_post else None, dres, keep, shares.cuda() if averaged else None, norm)
        k.residual_step(dev, *args, out)
        assert close(out, want, dtype) and close(dev, x, torch.float32) and close(dres, kept, torch.float32)
        rows = torch.tensor([4, 0, 4], dtype=torch.int32, device="cuda")
        dev, dres = h.cuda(), results.cuda()
        some = torch.empty((3, width), dtype=dtype, device="cuda")
        args = args[:2] + (dres,) + args[3:]
        k.residual_step(dev, *args, some, rows)
        assert torch.equal(some, out[[4, 0, 4]]) and torch.equal(dev.cpu(), h) and torch.equal(dres.cpu(), results)
        k.residual_step(dev, *args[:-1], None, None)                 # the flush: everything but the next norm
        assert close(dev, x, torch.float32) and close(dres, kept, torch.float32)


#: three requests in five steps: portions of unequal sizes (one of more than two rounds of the kernel), single tokens, a
#: request that sits steps out, a request that starts late in a slot of its own
STEPS = [([5, 1], [0, 0], [2, 0]), ([2, 3, 4], [5, 1, 0], [2, 0, 3]), ([1, 1], [7, 4], [2, 3]), ([1200, 1, 2], [8, 4, 5], [2, 0, 3]),
         ([1, 513, 70], [1208, 5, 7], [2, 0, 3])]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [1, 16, 90, 256])
def test_the_recurrence_over_unequal_requests(dtype, width):
    g = torch.Generator().manual_seed(width)
    bz, bx = torch.randn(width, generator=g) - 3.0, torch.randn(width, generator=g) * 0.5
    by_slot, want = {}, {}
    for slot in (0, 2, 3):
        raw = torch.randn((1250, 3 * width + 4), generator=g) * 1.5
        raw[17], raw[18] = 60.0, -60.0                                # gates that are open and shut to the last bit
        by_slot[slot] = raw
        z = plain.sigmoid((raw[:, 2:2 + width] + bz).double())
        S = plain.gated_average(z, (raw[:, 2 + width:2 + 2 * width] + bx).double())
        gate = raw[:, 2 + 2 * width:2 + 3 * width].double()
        want[slot] = S * gate * plain.sigmoid(gate)
    state = torch.zeros((4, width + 3), device="cuda")
    k = K()
    for lengths, starts, slots in STEPS:
        raw = torch.cat([by_slot[s][a:a + n] for n, a, s in zip(lengths, starts, slots)]).cuda()
        _, _, seqs = step_meta(lengths, starts, slots)
        out = torch.empty((raw.shape[0], width), dtype=dtype, device="cuda")
        single = all(n == 1 for n in lengths)
        k.channel_recurrence(raw, 2, 2 + width, 2 + 2 * width, bz.cuda(), bx.cuda(), seqs, len(lengths), single, state, out)
        expect = torch.cat([want[s][a:a + n] for n, a, s in zip(lengths, starts, slots)])
        assert close(out, expect, dtype, scale=0.1), (lengths, float((out.double().cpu() - expect).abs().max()))
    assert float(state[1].abs().max()) == 0.0 and float(state[:, width:].abs().max()) == 0.0


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [2, 45, 700])
def test_position_vectors_at_near_and_far_positions(dtype, width):
    g = torch.Generator().manual_seed(width)
    table = torch.randn((50, width), generator=g).to(dtype)
    tokens = torch.randint(0, 50, (6,), generator=g).to(torch.int32)
    positions = torch.tensor([0, 1, 77, 4095, 100003, 2000000], dtype=torch.int32)
    f = torch.tensor([10000.0 ** (-2.0 * i / width) for i in range((width + 1) // 2)], dtype=torch.float64)
    want = table.double()[tokens.long()] * 1.5
    angle = positions.double()[:, None] * f[None, :]
    want[:, 0::2] += torch.sin(angle)
    want[:, 1::2] += torch.cos(angle)[:, :width // 2]
    out = torch.empty((6, width), device="cuda")
    K().embed_positions(tokens.cuda(), positions.cuda(), table.cuda(), f.cuda(), out, 1.5)
    assert float((out.double().cpu() - want).abs().max()) < 2e-6


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows, n, kk", [(1, 48, 64), (8, 4608, 2048), (20, 10, 33), (40, 9000, 96), (64, 16640, 64), (200, 300, 96),
                                         (600, 1000, 45), (2100, 1100, 128)])
def test_the_product_with_xielu_behind_it(dtype, rows, n, kk):
    """Every kernel that serves it: few rows, a walk over column blocks, tiles of all sizes, operands that are not
    aligned; arguments near zero, where the terms cancel, and large ones of both signs."""
    g = torch.Generator().manual_seed(rows)
    x = torch.randn((rows, kk), generator=g).to(dtype)
    w = (torch.randn((n, kk), generator=g) * 2 / math.sqrt(kk)).to(dtype)
    w[:n // 3] *= 1e-3
    if rows > 1:
        w[n // 2] *= 20
    up, down = 1.3, 0.9
    z = x.double() @ w.double().T
    low = torch.clamp(z, max=0.0)
    want = torch.where(z > 0, up * z * z, down * (torch.expm1(low) - low)) + 0.5 * z
    out = torch.empty((rows, n), dtype=dtype, device="cuda")
    K().gemm_xielu(x.cuda(), w.cuda(), out, torch.tensor([up, down], device="cuda"))
    err = (out.double().cpu() - want).abs()
    rel = 3e-5 if dtype == torch.float32 else 8e-3
    assert bool((err <= rel * want.abs() + (2e-5 if dtype == torch.float32 else 2e-5)).all()), float((err / (want.abs() + 1e-3)).max())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_pass_behind_queries_without_a_latent(dtype):
    """Queries rounded as they are, the latent normalised into both kinds of page on scattered pages, the key's padding."""
    g = torch.Generator().manual_seed(5)
    t, qw, rank, pad, page = 7, 50, 20, 24, 4
    raw = torch.randn((t, qw + rank), generator=g)
    weight = 1 + 0.3 * torch.randn(rank, generator=g)
    tok_seq, tok_pos, seqs = step_meta([5, 2], [2, 7], [1, 0])
    table = torch.tensor([[6, 3, 5], [1, 4, 0]], dtype=torch.int32, device="cuda")
    keys = torch.full((8, 1, page, pad), 9.0, dtype=dtype, device="cuda")
    values = torch.full((8, 1, rank, page), 9.0, dtype=dtype, device="cuda")
    q = torch.empty((t, qw), dtype=dtype, device="cuda")
    K().latent_post(raw.cuda(), t, qw, rank, 0, pad, True, None, weight.cuda(), 1e-5, None, None, 0, 8, tok_seq, tok_pos, seqs, table,
                    q, keys, values, page)
    assert torch.equal(q.cpu(), raw[:, :qw].to(dtype))
    want = plain.rms_norm(raw[:, qw:].double(), weight.double(), 1e-5)
    rows = table.cpu()
    for i, (slot, pos) in enumerate([(1, 2), (1, 3), (1, 4), (1, 5), (1, 6), (0, 7), (0, 8)]):
        where = int(rows[slot, pos // page]), pos % page
        assert close(keys[where[0], 0, where[1], :rank], want[i], dtype)
        assert float(keys[where[0], 0, where[1], rank:].abs().max()) == 0.0
        assert torch.equal(values[where[0], 0, :, where[1]], keys[where[0], 0, where[1], :rank])
    assert int((keys == 9.0).all(dim=-1).sum()) == 8 * page - t


@pytest.mark.parametrize("activation", ["silu", "gelu", "gelu_tanh", "relu"])
def test_a_feed_forward_of_two_matrices_with_other_activations(activation):
    from lockstep_amd.config.base import PartSpec
    from lockstep_amd.engine.batch import Workspace
    from lockstep_amd.engine.runtime import Runtime
    from lockstep_amd.parts import build_part
    from lockstep_amd.weights.store import weights_from_dict

    g = torch.Generator().manual_seed(1)
    part = build_part(PartSpec("mlp", {"hidden_size": 32, "intermediate_size": 40, "activation": activation}), "m")
    tensors = {"m.up": torch.randn((40, 32), generator=g) * 0.3, "m.down": torch.randn((32, 40), generator=g) * 0.3}
    rt = Runtime("cuda:0", "float32")
    part.load(weights_from_dict(tensors, part.weight_specs(part.spec, "m"), {}), rt)

    class Step:
        n_tokens = 9
        workspace = Workspace(rt.device)

        def buf(self, *args):
            return self.workspace.get(*args)

    step = Step()
    step.rt = rt
    x = torch.randn((9, 32), generator=g)
    out = torch.empty((9, 32), device="cuda")
    part.forward(step, x.cuda(), out, accumulate=False)
    z = x.double() @ tensors["m.up"].double().T
    f = torch.nn.functional
    act = {"silu": f.silu, "gelu": f.gelu, "gelu_tanh": lambda v: f.gelu(v, approximate="tanh"), "relu": f.relu}[activation]
    assert close(out, act(z) @ tensors["m.down"].double().T, torch.float32)


# ---------------------------------------------------------------------------
# whole models
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("kind", list(SINGLE))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_each_mechanism_alone_whole_and_in_portions(models, kind, dtype):
    model, oracle, raw, page, _ = models(kind, dtype, table=SINGLE)
    tokens = random_tokens(75, raw["vocab"], seed=4)
    want = oracle.forward(tokens)
    for cuts in ([], [2, 31, 2, 17, 1, 1, 1], [1] * 75):
        cache = new_cache(model, page)
        err = rel_err(feed(model, cache, "r", tokens, cuts), want)
        print(f"{kind} {dtype} {cuts[:3]}: {err:.2e}")
        assert err < TOL[dtype], (kind, cuts[:3], err)
        cache.close("r")
        cache.audit()


@pytest.mark.parametrize("name", ["A", "B", "C"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_prompt_portions_and_token_by_token_agree_with_the_plain_model(models, name, dtype):
    model, oracle, raw, page, _ = models(name, dtype)
    tokens = random_tokens(150, raw["vocab"], seed=5)
    want = oracle.forward(tokens)
    runs = {}
    for label, cuts in (("whole", []), ("portions", [2, 47, 3, 16, 2, 33, 5, 1, 1, 2]), ("pairs", [2] * 75),
                        ("tail", [110] + [1] * 40), ("single", [1] * 150)):
        cache = new_cache(model, page)
        runs[label] = feed(model, cache, "r", tokens, cuts)
        err = rel_err(runs[label], want)
        print(f"{name} {dtype} {label}: {err:.2e}")
        assert err < tol(dtype, name), (name, label, err)
        cache.close("r")
        cache.audit()
    if dtype == "float32":              # the cuttings agree with each other far below the bound against the plain model
        for label in ("portions", "pairs", "tail", "single"):
            assert rel_err(runs[label], runs["whole"]) < tol(dtype, name), label


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B"])
def test_a_long_prompt_and_decoding_after_it(models, name, dtype):
    """A prompt of 700 tokens (many row blocks whose keys are dealt to runs, a recurrence over more than one round
    of its kernel), whole and cut at odd places, and twenty decoded tokens after it."""
    model, oracle, raw, page, _ = models(name, dtype)
    tokens = random_tokens(720, raw["vocab"], seed=13)
    want = oracle.forward(tokens)
    for cuts in ([700] + [1] * 20, [333, 2, 365] + [1] * 20):
        cache = new_cache(model, page, tokens=1024)
        err = rel_err(feed(model, cache, "r", tokens, cuts), want)
        print(f"{name} {dtype} {cuts[:3]}: {err:.2e}")
        assert err < TOL[dtype], (cuts[:3], err)
        cache.close("r")


@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_first_tokens_and_prompts_of_one_and_two_tokens(models, name):
    model, oracle, raw, page, _ = models(name)
    for n in (1, 2, 3, page, page + 1):
        tokens = random_tokens(n, raw["vocab"], seed=20 + n)
        cache = new_cache(model, page)
        assert rel_err(feed(model, cache, "r", tokens, []), oracle.forward(tokens)) < tol("float32", name), n


@pytest.mark.parametrize("name, dtype", [("A", "float32"), ("B", "float32"), ("C", "float32"), ("A", "bfloat16")])
def test_mixed_batches_of_unequal_requests_with_pages_and_slots_used_again(models, name, dtype):
    """Seven requests of unequal lengths through four slots and a pool that holds the live ones only: portions beside
    single tokens, requests that sit steps out, finished requests whose (poisoned) pages and state slots the next ones
    take.  Each request's logits equal those of the request alone."""
    model, oracle, raw, page, _ = models(name, dtype)
    lengths = [1, 23, 97, 150, 61, 2, 130]
    requests = {f"r{i}": random_tokens(n, raw["vocab"], seed=40 + i) for i, n in enumerate(lengths)}
    steps = make_mixed_trace(requests, seed=3, max_live=4, decode_tail=12, max_portion=29)
    assert any(len(s["entries"]) > 1 and {len(e["tokens"]) for e in s["entries"]} != {1} for s in steps)
    tokens = max_live_tokens(steps, round_to=page)
    cache = model.make_cache(num_pages=-(-tokens // page), page_size=page, max_requests=4,
                             max_tokens_per_request=max(lengths) + page, poison_on_free=True)
    got = replay_in_process(model, cache, steps)
    assert cache.free_slots == 4
    for rid, toks in requests.items():
        err = rel_err(got[rid], oracle.forward(toks))
        assert err < tol(dtype, name), (rid, err)


def test_only_the_wanted_rows_are_finished(models):
    """Logits asked for at a few places of several portions (the last step of the stream runs on those rows alone) are
    those of a step that asks for all, and the steps that follow are none the worse for it."""
    from lockstep_amd.engine.batch import StepEntry

    model, oracle, raw, page, _ = models("A")
    a, b = random_tokens(60, raw["vocab"], seed=1), random_tokens(45, raw["vocab"], seed=2)
    wa, wb = oracle.forward(a), oracle.forward(b)
    cache = new_cache(model, page)
    cache.open("a"), cache.open("b")
    assert model.step(cache, [StepEntry("a", a[:20], []), StepEntry("b", b[:9], [])]) is None
    got = model.step(cache, [StepEntry("b", b[9:30], [20, 3]), StepEntry("a", a[20:21], [0])])
    assert rel_err(got.cpu(), torch.stack([wb[29], wb[12], wa[20]])) < TOL["float32"]
    got = model.step(cache, [StepEntry("a", a[21:60], [38]), StepEntry("b", b[30:45], [0, 14])])
    assert rel_err(got.cpu(), torch.stack([wa[59], wb[30], wb[44]])) < TOL["float32"]


# ---------------------------------------------------------------------------
# far keys, page borders, state
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("kind", ["latent", "latent_2", "shared"])
@pytest.mark.parametrize("page", [8, 16])
def test_single_keys_far_away_and_at_page_borders(tmp_path, monkeypatch, kind, page):
    """Peaked attention, where one key often holds most of a row's weight.  Controls: losing any one key among the first
    ones, at a page's border, or next to the query moves the plain logits far behind it by many times the bound, so an
    engine that agrees in prompts, portions that end at the borders, and decoding has lost none."""
    from lockstep_amd import load_model

    n = 200
    raw = json.loads(json.dumps(SINGLE[kind]["raw"]))
    for layer in raw["layers"]:
        layer["mixer"]["scale"] = 1.5
    tensors = make_tensors(raw, seed=21, spread=1.3)
    model = load_model(write_model(tmp_path / "m", raw, tensors), dtype="float32")
    oracle = plain.PlainTukavik(raw, tensors)
    tokens = random_tokens(n, raw["vocab"], seed=6)
    want = oracle.forward(tokens)
    whole = plain.causal_attention

    def without(lost):
        def attention(q, k, v, scale):
            s = (q @ k.T) * scale
            seen = torch.tril(torch.ones_like(s, dtype=torch.bool))
            seen[lost + 1:, lost] = False
            return torch.softmax(s.masked_fill(~seen, -math.inf), dim=-1) @ v
        return attention

    for lost in (0, 1, page - 1, page, 2 * page - 1, 2 * page, 127, 128):
        monkeypatch.setattr(plain, "causal_attention", without(lost))
        assert rel_err(oracle.forward(tokens)[lost + 30:], want[lost + 30:]) > 30 * TOL["float32"], lost
    monkeypatch.setattr(plain, "causal_attention", whole)
    for cuts in ([], [page, page, page - 1, 2, page + 1], [page - 1, 1, 1, 2 * page, 2], [1] * n, [130] + [1] * 70):
        cache = new_cache(model, page, tokens=256)
        err = rel_err(feed(model, cache, "r", tokens, cuts), want)
        print(f"{kind} {page} {cuts[:3]}: {err:.2e}")
        assert err < TOL["float32"], (kind, cuts[:3], err)
        cache.close("r")
        cache.audit()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_far_token_that_only_the_state_still_holds(tmp_path, dtype):
    """Two recurrences and no attention: the third token of 300 still shows in the last logits (control), through the
    state that prompt portions and decoded tokens carried."""
    from lockstep_amd import load_model

    raw = config(48, 40, [dense(recurrence(64), 32), bare(recurrence(24))])
    tensors = make_tensors(raw, seed=22)
    for i in range(2):
        tensors[f"l{i}.mix.z.b"] = torch.full_like(tensors[f"l{i}.mix.z.b"], -4.5)      # (a long memory)
    model = load_model(write_model(tmp_path / "m", raw, tensors), dtype=dtype)
    oracle = plain.PlainTukavik(raw, tensors)
    tokens = random_tokens(300, raw["vocab"], seed=7)
    want = oracle.forward(tokens)
    changed = list(tokens)
    changed[2] = (tokens[2] + 1) % raw["vocab"]
    assert rel_err(oracle.forward(changed)[-20:], want[-20:]) > 20 * TOL["float32"]
    for cuts in ([], [100, 2, 150] + [1] * 48, [250] + [1] * 50):
        cache = new_cache(model, 8, tokens=384)
        err = rel_err(feed(model, cache, "r", tokens, cuts), want)
        assert err < TOL[dtype], (cuts[:3], err)
        cache.close("r")


def test_a_latent_of_128_elements_on_both_kinds_of_layer(tmp_path):
    """A latent of a real model's size (the staged kernel for prompt portions), read by a second layer, in bfloat16."""
    from lockstep_amd import load_model

    raw = config(128, 96, [dense(latent(8, 32, 48, kv_rank=128, scale=0.2), 64),
                           dense(latent(4, 48, 32, kv_rank=128, scale=0.15, q_rank=64, kv_from=0), 64)])
    tensors = make_tensors(raw, seed=8)
    oracle = plain.PlainTukavik(raw, tensors)
    tokens = random_tokens(300, raw["vocab"], seed=7)
    want = oracle.forward(tokens)
    folder = write_model(tmp_path / "m", raw, tensors)
    for dtype in ("float32", "bfloat16"):
        model = load_model(folder, dtype=dtype)
        for cuts in ([290] + [1] * 10, [40, 2, 150, 17]):
            cache = new_cache(model, 16, tokens=320)
            err = rel_err(feed(model, cache, "r", tokens, cuts), want)
            print(f"128 {dtype} {cuts[:3]}: {err:.2e}")
            assert err < TOL[dtype], (dtype, cuts[:3], err)


# ---------------------------------------------------------------------------
# long decoding, generation, the programs
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_long_decoding_of_two_requests_through_replayed_graphs(models, name):
    from lockstep_amd.engine.batch import StepEntry

    model, oracle, raw, page, _ = models(name)
    a, b = random_tokens(230, raw["vocab"], seed=8), random_tokens(215, raw["vocab"], seed=9)
    cache = new_cache(model, page, tokens=512)
    cache.open("a"), cache.open("b")
    model.step(cache, [StepEntry("a", a[:30], []), StepEntry("b", b[:15], [])])
    replays = model.graph_replays
    rows = {"a": [], "b": []}
    for t in range(200):
        logits = model.step(cache, [StepEntry("a", [a[30 + t]], [0]), StepEntry("b", [b[15 + t]], [0])])
        rows["a"].append(logits[0].cpu()), rows["b"].append(logits[1].cpu())
    assert model.graph_replays - replays >= 150
    assert rel_err(torch.stack(rows["a"]), oracle.forward(a)[30:]) < tol("float32", name)
    assert rel_err(torch.stack(rows["b"]), oracle.forward(b)[15:]) < tol("float32", name)


@pytest.mark.parametrize("name", ["A", "B"])
def test_greedy_generation_through_the_scheduler_and_the_single_prompt_entry_point(models, name):
    from lockstep_amd import LLM, Request

    _, oracle, raw, page, folder = models(name, seed=12)
    prompts = [random_tokens(n, raw["vocab"], seed=60 + n) for n in (5, 41, 18)]
    want = [oracle.generate_greedy(p, 24) for p in prompts]
    llm = LLM(folder, dtype="float32", num_pages=64, page_size=page)
    got = llm.generate([Request(uid=f"r{i}", prompt=p, max_new_tokens=24) for i, p in enumerate(prompts)])
    assert [got[f"r{i}"] for i in range(3)] == want
    alone, _ = llm.generate_greedy(prompts[1], 24)
    assert alone == want[1]
    half = LLM(folder, dtype="bfloat16", num_pages=64, page_size=page)
    tokens = half.generate([Request(uid="x", prompt=prompts[0], max_new_tokens=8)])["x"]
    assert len(tokens) == 8 and tokens[:2] == want[0][:2]


def test_trace_replay_program_on_a_model_folder(models, tmp_path):
    """bin/trace_run as a subprocess on a Tukavik folder: a mixed schedule through four slots."""
    _, oracle, raw, page, folder = models("A")
    requests = {f"q{i}": random_tokens(n, raw["vocab"], seed=80 + i) for i, n in enumerate([40, 3, 77, 52, 19])}
    steps = make_mixed_trace(requests, seed=5, max_live=4, decode_tail=6, max_portion=19)
    out = tmp_path / "out"
    proc = subprocess.Popen([sys.executable, str(ROOT / "bin" / "trace_run"), "--model", str(folder), "--dtype", "float32",
                             "--out", str(out), "--max-tokens", str(max_live_tokens(steps)), "--page-size", str(page)],
                            stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
    try:
        for step in steps:
            proc.stdin.write(json.dumps(step) + "\n")
            proc.stdin.flush()
            assert proc.stdout.readline().strip() == f"done {step['step']}"
        proc.stdin.close()
        assert proc.wait(timeout=60) == 0
    finally:
        if proc.poll() is None:
            proc.kill()
    rows: dict = {}
    for step in steps:
        data = np.fromfile(out / f"{step['step']}.f32", dtype="<f4").reshape(-1, raw["vocab"])
        at = 0
        for e in step["entries"]:
            rows.setdefault(e["id"], []).append(data[at:at + len(e["want"])])
            at += len(e["want"])
    for rid, toks in requests.items():
        assert rel_err(np.concatenate(rows[rid]), oracle.forward(toks)) < TOL["float32"], rid
