"""Fuvevik through the engine against the plain implementation (``plain_fuvevik.py``): every mechanism alone and all
together, whole prompts against portions and single tokens, unequal batches against each request alone, pages and slots
that are used again, keys far back, at the edges of pages and of the kernels' tiles of 64 keys, positions just before, on
and behind every step of the query factor, in prompts and in decoding, the first tokens of a sequence, long decoding, and
greedy generation through ``Engine``, the command line and the trace program.

Models are written with the random-weights mode in bfloat16 (so that both compute types see the same numbers as the
plain implementation) with larger matrices than the architecture's rule draws, so that a mixer or feed-forward that
went wrong moves the logits by far more than the tolerance; where random weights would still hide a fault (one key
among hundreds, a sink, a step of the query factor) the test makes the inputs or the constants that show it.
"""
import functools
import json
import os
import shutil
import tempfile

import numpy as np
import pytest
import torch

import fuvevik_configs as Z
import plain_fuvevik as P
from gpu_common import random_tokens

pytestmark = pytest.mark.gpu

_root = None
_folders = {}


def folder_of(name: str, seed: int = 11) -> str:
    global _root
    key = (name, seed)
    if key not in _folders:
        import nanoinfer_amd  # noqa: F401
        from nanoinfer_amd.weights.loader import make_random_model
        if _root is None:
            _root = tempfile.mkdtemp(prefix="fuvevik-tests-")
            import atexit
            atexit.register(shutil.rmtree, _root, ignore_errors=True)
        _folders[key] = make_random_model(os.path.join(_root, f"{name}-{seed}-{len(_folders)}"), Z.ALL[name], seed,
                                          dtype="bfloat16", matrix_std=0.12)
    return _folders[key]


@functools.lru_cache(maxsize=None)
def _model(folder: str):
    return P.read_model_folder(folder)


@functools.lru_cache(maxsize=None)
def _plain(folder: str, tokens: tuple):
    cfg, w = _model(folder)
    margins = np.full(len(tokens), np.inf)
    return torch.from_numpy(P.forward(cfg, w, list(tokens), margins=margins)), torch.from_numpy(margins)


class Plain(torch.Tensor):
    """The plain logits of a sequence, with ``margins`` [tokens]: the smallest gap by which a router chose for each."""


def plain(folder: str, tokens: tuple) -> torch.Tensor:
    logits, margins = _plain(folder, tokens)
    out = logits.as_subclass(Plain)
    out.margins = margins
    return out


def runner_for(folder, dtype, **kw):
    from nanoinfer_amd.engine.runner import ModelRunner
    kw.setdefault("page_size", 8)
    kw.setdefault("max_tokens", 2048)
    kw.setdefault("max_requests", 4)
    return ModelRunner(folder, dtype=dtype, **kw)


def replay(runner, requests, steps):
    """Run ``steps`` (each a dict request -> number of its next tokens), asking for every row; returns
    request -> logits [tokens, vocab].  A request ends with its last token."""
    from nanoinfer_amd.engine.runner import StepEntry
    done = {r: 0 for r in requests}
    rows = {r: [] for r in requests}
    for counts in steps:
        entries = [StepEntry(r, list(requests[r][done[r]:done[r] + c]), list(range(c))) for r, c in counts.items()]
        out = runner.step(entries, end=[r for r, c in counts.items() if done[r] + c == len(requests[r])])
        at = 0
        for r, c in counts.items():
            rows[r].append(out[at:at + c].clone())
            at += c
            done[r] += c
    assert all(done[r] == len(requests[r]) for r in requests)
    return {r: torch.cat(v) for r, v in rows.items()}


def all_pages_free(cache) -> bool:
    return all(g.pages.num_free == g.pages.num_pages for g in cache.groups)


def cuts(n, sizes):
    out, i = [], 0
    while n > 0:
        c = min(n, sizes[i % len(sizes)])
        out.append(c)
        n -= c
        i += 1
    return out


DTYPES = ["float32", "bfloat16"]

# Float32 is the sharp comparison, row by row against the row's own largest logit: at most one row in fifty beyond
# 2e-5 and none beyond 1e-4.  bfloat16 is judged row by row by the root mean square of the difference over the
# vocabulary (its mean taken off) against the root mean square of the plain logits: the median row within 2.5e-2, at
# most one row in ten beyond 5e-2, none beyond 0.15.  The models are drawn with large matrices on purpose, so rounding
# weighs more than in a trained model; a fault (a key too many, a forgotten sink, an expert that was not chosen) moves
# many rows by the size of the logits themselves.  A router chooses by comparing scores, and a score that bfloat16
# rounding of its input moves by a few thousandths can fall on the other side of its neighbour: the token then runs
# another expert in either implementation with equal right.  The plain implementation says by how little every token's
# choices were made; in bfloat16 the rows of tokens that chose by less than ``CLOSE_CALL`` are held to the median and to
# the count of rows beyond 5e-2, not to the bound on the worst row.
F32_ROW, F32_WORST = 2e-5, 1e-4
BF16_MEDIAN, BF16_ROW, BF16_WORST = 2.5e-2, 5e-2, 0.15
CLOSE_CALL, CLOSE_CALL_F32 = 0.03, 1e-5
worst_row = {"float32": 0.0, "bfloat16": 0.0}


def assert_close(got, want, dtype, what=""):
    assert tuple(got.shape) == tuple(want.shape), what
    diff = got.double().cpu() - want
    margins = getattr(want, "margins", None)
    if dtype == "float32":
        per_row = diff.abs().max(dim=-1).values / want.abs().max(dim=-1).values
        if margins is not None:         # a choice made by less than float32 rounding moves a score
            per_row = torch.where(margins < CLOSE_CALL_F32, torch.zeros_like(per_row), per_row)
        worst_row[dtype] = max(worst_row[dtype], float(per_row.max()))
        over = int((per_row > F32_ROW).sum())
        assert over <= max(1, per_row.numel() // 50), f"{what}: {over} of {per_row.numel()} rows are off by more than {F32_ROW} (float32)"
        assert float(per_row.max()) <= F32_WORST, f"{what}: row {int(per_row.argmax())} is off by {float(per_row.max()):.3e} (float32)"
        return
    diff = diff - diff.mean(dim=-1, keepdim=True)
    per_row = diff.pow(2).mean(dim=-1).sqrt() / want.pow(2).mean().sqrt()
    worst_row[dtype] = max(worst_row[dtype], float(per_row.max()))
    assert float(per_row.median()) <= BF16_MEDIAN, f"{what}: the median row is off by {float(per_row.median()):.3e} (bfloat16)"
    over = int((per_row > BF16_ROW).sum())
    assert over <= max(1, per_row.numel() // 10), f"{what}: {over} of {per_row.numel()} rows are off by more than {BF16_ROW} (bfloat16)"
    if margins is not None:
        per_row = torch.where(margins < CLOSE_CALL, torch.zeros_like(per_row), per_row)
    assert float(per_row.max()) <= BF16_WORST, f"{what}: row {int(per_row.argmax())} is off by {float(per_row.max()):.3e} (bfloat16)"


def test_zz_report_worst_rows():
    print(f"worst rows of the Fuvevik comparisons: {worst_row}")


# ------------------------------------------------------------------ every mechanism alone

ALONE = ["attn_only", "attn_plain", "attn_narrow", "dense_only", "moe_only", "moe_bare", "moe_identity", "moe_all", "moe_many"]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ALONE)
def test_one_mechanism_whole_prompt_and_token_by_token(name, dtype):
    """A model of one layer: a whole prompt, then the same tokens as a short portion followed by single tokens, both equal
    to the plain implementation row by row."""
    folder = folder_of(name)
    toks = random_tokens(Z.ALL[name]["vocab"], 75, 5)
    want = plain(folder, toks)
    runner = runner_for(folder, dtype)
    got = replay(runner, {"w": toks}, [{"w": len(toks)}])["w"]
    assert_close(got, want, dtype, f"{name} whole")
    got = replay(runner, {"d": toks}, [{"d": 3}] + [{"d": 1}] * (len(toks) - 3))["d"]
    assert_close(got, want, dtype, f"{name} token by token")
    assert not runner.cache.live_requests()


# ------------------------------------------------------------------ the whole design, every schedule

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "shared_kv", "odd_sizes", "many_streams", "five_streams"])
def test_portions_of_several_sizes_down_to_two_tokens(name, dtype):
    folder = folder_of(name)
    toks = random_tokens(Z.ALL[name]["vocab"], 150, 21)
    want = plain(folder, toks)
    runner = runner_for(folder, dtype)
    for sizes in ([150], [2], [37, 2, 23, 3], [64, 1, 1, 17], [5, 8, 16, 1]):
        got = replay(runner, {"p": toks}, [{"p": c} for c in cuts(len(toks), sizes)])["p"]
        assert_close(got, want, dtype, f"{name} in portions of {sizes}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("graphs", [True, False])
def test_unequal_requests_in_one_batch_equal_each_alone_and_slots_are_used_again(dtype, graphs):
    """Six requests of 1 to 130 tokens through a pool that holds three at a time and too few pages for all: portions
    beside single tokens, requests that pause for a step, pages and slots that the next request takes over as they are.
    Every row equals the plain implementation of its request alone."""
    name = "mixed"
    folder = folder_of(name)
    vocab = Z.ALL[name]["vocab"]
    lengths = {"a": 130, "b": 1, "c": 47, "d": 80, "e": 2, "f": 66}
    requests = {r: random_tokens(vocab, n, 40 + i) for i, (r, n) in enumerate(lengths.items())}
    runner = runner_for(folder, dtype, max_tokens=8 * 36, max_requests=3, use_graphs=graphs)
    steps = [{"a": 30}, {"a": 29, "b": 1, "c": 2}, {"a": 1, "c": 16}, {"c": 1, "a": 7}, {"a": 1, "c": 1}, {"a": 1, "c": 27},
             {"a": 61}]
    steps += [{"d": 40, "e": 1}, {"e": 1, "d": 1}, {"d": 39}]
    steps += [{"f": 64}, {"f": 1}, {"f": 1}]
    got = replay(runner, requests, steps)
    for r, toks in requests.items():
        assert_close(got[r], plain(folder, toks), dtype, f"request {r}")
    runner.cache.check()
    assert not runner.cache.live_requests() and all_pages_free(runner.cache)
    assert runner.cache.slots.num_free == 3


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_in_a_batch_of_recorded_steps(dtype):
    """Three requests decode 160 tokens each side by side after prompts of unequal length, across many page edges, every
    step of the query factors and two edges of the attention's tiles of 64 keys, in recorded steps."""
    name = "mixed"
    folder = folder_of(name)
    vocab = Z.ALL[name]["vocab"]
    prompts = {"x": 5, "y": 61, "z": 30}
    requests = {r: random_tokens(vocab, n + 160, 70 + i) for i, (r, n) in enumerate(prompts.items())}
    runner = runner_for(folder, dtype)
    got = replay(runner, requests, [dict(prompts)] + [{r: 1 for r in prompts}] * 160)
    assert any(key[0] == "d" for key in runner._recorded), "the decode steps were not recorded"
    for r, toks in requests.items():
        assert_close(got[r], plain(folder, toks), dtype, f"request {r}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_first_tokens_of_a_sequence(dtype):
    """Requests of one and of two tokens, and the first rows of a longer one, on the slot and the pages that a longer
    request has just left: nothing of the request before shows."""
    name = "mixed"
    folder = folder_of(name)
    vocab = Z.ALL[name]["vocab"]
    runner = runner_for(folder, dtype, max_requests=1, max_tokens=96)
    long = random_tokens(vocab, 90, 3)
    replay(runner, {"long": long}, [{"long": 90}])
    for n in (1, 2, 5):
        toks = random_tokens(vocab, n, 100 + n)
        got = replay(runner, {"s": toks}, [{"s": 1}] * n)["s"]
        assert_close(got, plain(folder, toks), dtype, f"{n} first tokens")
    toks = random_tokens(vocab, 6, 77)
    assert_close(replay(runner, {"s": toks}, [{"s": 6}])["s"], plain(folder, toks), dtype, "a first portion")


@pytest.mark.parametrize("dtype", DTYPES)
def test_layer_by_layer_against_the_plain_stream(dtype):
    """The stream behind every layer, through ``Model.tap``."""
    folder = folder_of("mixed")
    cfg, w = _model(folder)
    toks = list(random_tokens(cfg["vocab"], 40, 8))
    want, margins = [], np.full(len(toks), np.inf)
    P.forward(cfg, w, toks, layers_out=want, margins=margins)
    sure = margins >= (CLOSE_CALL_F32 if dtype == "float32" else CLOSE_CALL)      # tokens whose experts were chosen beyond doubt
    assert sure.sum() >= len(toks) // 3
    runner = runner_for(folder, dtype, use_graphs=False)
    got = []
    runner.model.tap = lambda i, h: got.append(h.detach().double().cpu())
    replay(runner, {"t": tuple(toks)}, [{"t": len(toks)}])
    assert len(got) == len(want) == len(cfg["layers"])
    tol = 2e-5 if dtype == "float32" else 6e-2
    for i, (a, b) in enumerate(zip(got, want)):
        err = float((a - torch.from_numpy(b)).abs()[sure].max() / np.abs(b).max())
        assert err <= tol, f"layer {i}: {err:.3e}"


# ------------------------------------------------------------------ far keys, the sink and the query factor, made to show

@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,dk,dv,page,temp", [(6, 2, 16, 32, 8, (0.7, 19)), (4, 4, 32, 16, 16, (1.5, 64)), (3, 1, 24, 24, 4, (0.5, 1)),
                                                 (5, 5, 16, 16, 8, None), (8, 1, 112, 64, 8, (0.3, 100)), (2, 1, 20, 12, 8, (0.9, 33)),
                                                 (16, 2, 64, 64, 16, (0.2, 128)), (3, 1, 48, 160, 8, (0.4, 63)),
                                                 (20, 1, 32, 32, 4, (0.3, 40))])
def test_far_keys_the_sink_and_the_query_factor_in_both_attention_kernels(H, G, dk, dv, page, temp, dtype):
    """The attention alone over scattered pages, with one key a query made to stand out: the first key, keys far back, at
    the edges of pages and of the kernels' tiles of 64, and the query's own.  The standing-out score is of the size of the
    heads' sinks (which run from no weight to most of it), so a sink that is left out, counted a run too often or scaled
    shows in every row, and so does a query factor that steps one position off.  Prompt portions (the matrix cores where
    they take the sizes, else the vector units) and single tokens with the keys cut into runs must both give the
    written-out softmax, as it is, with a gate a channel and with a gate a head."""
    from nanoinfer_amd import kernels as K
    from nanoinfer_amd.kernels import stream
    dev = torch.device("cuda")
    T = 300
    g = torch.Generator().manual_seed(3)
    k = torch.randn(T, G, dk, generator=g) * 0.1
    q = torch.randn(T, H, dk, generator=g) * 0.1
    for i in range(T):
        places = [0, i // 2, i - 63, i - 64, i - 65, i // page * page, i // page * page - 1, i]
        j = places[i % len(places)]
        if 0 <= j <= i:
            q[i] = k[j, torch.arange(H) // (H // G)] * (30.0 / max(float(k[j].pow(2).sum(-1).max()), 1e-3))
    scale = 0.5
    sink = torch.linspace(-10.0, 40.0, H)            # the standing-out score is about 15 times the query factor
    qd, kd, vd = q.to(dtype), k.to(dtype), torch.randn(T, G, dv, generator=g).to(dtype)
    factor = P.temperature(np.arange(T), None if temp is None else dict(zip(("coef", "every"), temp)))

    def written_out(factor):
        out = np.zeros((T, H, dv))
        for h in range(H):
            scores = qd[:, h].double().numpy() @ kd[:, h // (H // G)].double().numpy().T * scale * factor[:, None]
            out[:, h] = P.sink_softmax(scores, float(sink[h])) @ vd[:, h // (H // G)].double().numpy()
        return torch.from_numpy(out.reshape(T, -1))

    want = written_out(factor)
    before = 3                                        # columns that belong to nobody
    gates = torch.randn(T, before + H * dv + 2, generator=g)
    factors = {None: 1.0, 1: torch.sigmoid(gates[:, before:before + H * dv].double()),
               dv: torch.sigmoid(gates[:, before:before + H].double()).repeat_interleave(dv, dim=1)}
    if temp is not None and temp[1] > 1:                                  # rows do depend on where the factor steps
        shifted = P.temperature(np.arange(T) - 1, dict(zip(("coef", "every"), temp)))
        moved = (written_out(shifted) - want).abs().max(dim=1).values / want.abs().max()
        assert float(moved[temp[1] - 1]) > 5e-2 or float(moved.max()) > 5e-2
    n_pages = (T + page - 1) // page
    perm = torch.randperm(n_pages + 5, generator=torch.Generator().manual_seed(1))[:n_pages]
    kpool = torch.full((n_pages + 5, G, page, dk), float("nan"), dtype=dtype)
    vpool = torch.full((n_pages + 5, G, page, dv), float("nan"), dtype=dtype)
    for t in range(T):
        kpool[perm[t // page], :, t % page] = kd[t]
        vpool[perm[t // page], :, t % page] = vd[t]
    kpool, vpool = kpool.to(dev), vpool.to(dev)
    pages = perm.to(torch.int32).view(1, -1).to(dev)
    qrows = qd.reshape(T, H * dk).contiguous().to(dev)
    positions = torch.arange(T, dtype=torch.int32, device=dev)
    sink_dev = sink.to(dev)
    coef, every = temp or (0.0, 0)
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    group = H // G

    def gate(rows, every):
        return None if every is None else (gates[rows].contiguous().to(dev), before, every)

    def check(out, rows, every, what):
        full = want * factors[every]
        err = float((out.double().cpu() - full[rows]).abs().max() / full.abs().max())
        assert err <= tol, f"{what}, gate every {every}: {err:.3e}"

    for start in (0, 100, 203):
        n = T - start
        for wide in (True, False):
            rows_per = stream.bias_attention_mfma_rows(dk, dv) if wide else stream.bias_attention_rows()
            if not rows_per:
                continue
            heads = min(group, rows_per)
            tiles = torch.tensor(K.build_q_tiles([0], [n], [T], max(1, rows_per // heads)), dtype=torch.int32).view(-1, 4).to(dev)
            fn = stream.bias_attention_mfma if wide else stream.bias_attention
            for per in (None, 1, dv):
                out = torch.empty(n, H * dv, dtype=dtype, device=dev)
                fn(qrows[start:].contiguous(), kpool, vpool, pages, tiles, positions[start:].contiguous(), None, out, H, scale, coef, every,
                   heads, sink=sink_dev, gate=gate(slice(start, T), per))
                check(out, slice(start, T), per, f"portion from {start}, {'matrix cores' if wide else 'vector units'}")
    heads = min(group, stream.bias_attention_rows())
    edges = [] if not every else [m * every + o for m in (1, 2) for o in (-2, -1, 0)]
    for pos in [0, 1, 63, 64, 65, 127, 128, 200, 299] + edges:
        if not 0 <= pos < T:
            continue
        tiles = torch.tensor(K.build_q_tiles([0], [1], [pos + 1], 1), dtype=torch.int32).view(-1, 4).to(dev)
        for runs, per in ((1, None), (1, 1), (3, None), (3, dv), (8, 1), (8, dv)):
            out = torch.empty(1, H * dv, dtype=dtype, device=dev)
            ws = torch.empty(H * runs * (dv + 2), dtype=torch.float32, device=dev) if runs > 1 else None
            stream.bias_attention(qrows[pos:pos + 1].contiguous(), kpool, vpool, pages, tiles, positions[pos:pos + 1].contiguous(), None,
                                  out, H, scale, coef, every, heads, runs, ws, 4, sink=sink_dev, gate=gate(slice(pos, pos + 1), per))
            check(out, slice(pos, pos + 1), per, f"single token at {pos} in {runs} runs")


@pytest.mark.parametrize("dtype", DTYPES)
def test_steps_of_the_query_factor_in_a_whole_model(dtype):
    """A model whose scores are sharp enough for the query factor to decide, stepping every 19 positions in one layer and
    every 64 in the layer that reads its keys: prompts that end, portions that start and single tokens that fall just
    before, on and just behind every step, the edges of pages (8) and of the kernels' tiles of 64 keys."""
    folder = folder_of("sharp")
    toks = random_tokens(Z.SHARP["vocab"], 230, 9)
    want = plain(folder, toks)
    runner = runner_for(folder, dtype)
    for start in (2, 17, 18, 19, 20, 37, 38, 62, 63, 64, 65, 127, 128, 129):
        rest = len(toks) - start
        steps = [{"k": start}] + [{"k": 1}] * 3 + [{"k": c} for c in cuts(rest - 3, [62, 2, 1, 64, 3])]
        assert_close(replay(runner, {"k": toks}, steps)["k"], want, dtype, f"first portion of {start}")
    got = replay(runner, {"k": toks}, [{"k": 10}] + [{"k": 1}] * (len(toks) - 10))["k"]
    assert_close(got, want, dtype, "decoded past every step")
    # the rows do depend on where the factor steps
    base, w = _model(folder)
    for layer, delta in ((0, 1), (0, -1), (1, 1), (1, -1)):
        other = json.loads(json.dumps(base))
        other["layers"][layer]["mixer"]["q_temp"]["every"] += delta
        moved = np.abs(P.forward(other, w, list(toks[:130])) - want[:130].numpy()).max() / np.abs(want.numpy()).max()
        assert moved > 1e-2, (layer, delta, moved)


# ------------------------------------------------------------------ the kernels of the design alone

@pytest.mark.parametrize("out", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,d,s,n", [(1, 64, 2, 1), (9, 2048, 4, 3), (70, 50, 3, 2), (33, 40, 1, 1), (5, 36, 5, 1), (130, 72, 8, 2),
                                     (3, 37, 11, 1), (2, 16, 32, 4), (2, 12800, 4, 1), (300, 96, 3, 1)])
def test_streams_are_mixed_summed_and_normed_in_one_pass(T, d, s, n, out):
    """``link_streams``: from one row a token (all streams equal) and from its streams, in place and to another tensor,
    with and without a sublayer's output before it, with and without the next sublayer's weights and norm, for all rows
    and for some."""
    from nanoinfer_amd import kernels as K
    dev = torch.device("cuda")
    g = torch.Generator().manual_seed(T + d + s)
    x = torch.randn(T, s, d, generator=g)
    y = torch.randn(n, T, d, generator=g)
    mix, adds, reads = torch.randn(s, s, generator=g), torch.randn(s, generator=g), torch.randn(s, generator=g)
    w = 1.0 + 0.3 * torch.randn(d, generator=g)
    eps = 1e-5
    norm = lambda u: P.rms(u, eps) * w.double().numpy()
    hc = {"h.in": reads.double().numpy(), "h.out": adds.double().numpy(), "h.mix": mix.double().numpy()}
    tol = 2e-5 if out == torch.float32 else 8e-3
    on = lambda t: t.to(dev)
    mixd, addsd, readsd, wd, yd = map(on, (mix, adds, reads, w, y))

    def close(got, want, tol, what):
        err = float(np.abs(got.double().cpu().numpy() - want).max() / max(np.abs(want).max(), 1e-6))
        assert err <= tol, f"{what}: {err:.3e}"

    for equal in (True, False):
        start = x[:, :1].expand(T, s, d) if equal else x
        streams = start.double().numpy().transpose(1, 0, 2)
        h0 = on(start[:, 0].contiguous() if equal else start.contiguous())
        v = torch.empty(T, d, dtype=out, device=dev)
        K.link_streams(h0, s, None, None, None, readsd, wd, eps, v)
        close(v, norm(P.sublayer_input(streams, hc, "h.")), tol, f"equal={equal}: the first sublayer's input")
        moved = P.sublayer_output(streams, y.double().sum(0).numpy(), hc, "h.")
        for in_place in ((False,) if equal else (False, True)):
            h = h0.clone()
            target = h if in_place else torch.full((T, s, d), float("nan"), device=dev)
            K.link_streams(h, s, yd if n > 1 else yd[0], mixd, addsd, readsd, wd, eps, v, h_out=target)
            close(target, moved.transpose(1, 0, 2), 5e-6, f"equal={equal}, in place {in_place}: the new streams")
            close(v, norm(P.sublayer_input(moved, hc, "h.")), tol, "the next sublayer's input")
            if not in_place:
                assert torch.equal(h, h0)
        total = torch.empty(T, d, dtype=torch.float32, device=dev)
        K.link_streams(h0, s, yd, mixd, addsd, None, None, 0.0, total)
        close(total, moved.sum(axis=0), 5e-6, "the sum of the streams")
        rows = torch.tensor([T - 1, 0, T // 2], dtype=torch.int32)
        picked = torch.empty(3, d, dtype=out, device=dev)
        K.link_streams(h0, s, yd, mixd, addsd, None, wd, eps, picked, rows=on(rows))
        close(picked, norm(moved.sum(axis=0))[rows.numpy()], tol, "some rows, normed")


def test_streams_that_do_not_fit_are_refused():
    from nanoinfer_amd import kernels as K
    dev = torch.device("cuda")
    h, v = torch.zeros(2, 3, 8, device=dev), torch.zeros(2, 8, device=dev)
    w = torch.ones(3, device=dev)
    with pytest.raises(K.KernelError):
        K.link_streams(h, 4, None, None, None, torch.ones(4, device=dev), None, 0.0, v)          # three streams are not four
    with pytest.raises(K.KernelError):
        K.link_streams(h, 3, None, None, None, w, None, 0.0, v, h_out=h)                          # nothing has moved
    with pytest.raises(K.KernelError):
        K.link_streams(h, 3, v, torch.ones(3, 3, device=dev), w, w, None, 0.0, v[:1], h_out=h, rows=torch.zeros(1, dtype=torch.int32, device=dev))
    big = torch.zeros(1, 40000, device=dev)
    with pytest.raises(K.KernelError):
        K.link_streams(big, 2, None, None, None, torch.ones(2, device=dev), big[0], 1e-5, torch.zeros_like(big))


@pytest.mark.parametrize("E,top", [(15, 4), (6, 1), (7, 7), (64, 8), (70, 6), (300, 70), (1, 1)])
def test_the_router_with_shares_of_all_and_a_correction(E, top):
    """Outputs chosen by their share of the softmax over all plus a correction, weighed by the chosen shares over their
    sum: against the plain router, for corrections large enough to reorder the outputs and to make choice scores negative."""
    from nanoinfer_amd import kernels as K
    dev = torch.device("cuda")
    g = torch.Generator().manual_seed(E * 7 + top)
    T = 97
    z = torch.randn(T, E, generator=g) * 2.0
    z[0] += 200.0                                     # only differences count
    corr = torch.randn(E, generator=g) * (1.0 / E)
    mlp = {"router": {"experts": E, "top": top}}
    w = {"l0.mlp.router": np.eye(E), "l0.mlp.correction": corr.double().numpy()}
    want_chosen, want_w = P.route(z.double().numpy(), mlp, w, "l0.")
    chosen, mix, dense = K.route_top(z.to(dev), top, mix_all=True, scoring="softmax_share", correction=corr.to(dev))
    chosen, mix, dense = chosen.cpu().numpy(), mix.cpu().numpy(), dense.cpu().numpy()
    same = [t for t in range(T) if chosen[t].tolist() == want_chosen[t].tolist()]
    assert len(same) >= T - 2 - T * top // 500        # a close call between two float32 scores may fall the other way
    for t in same:
        assert np.allclose(mix[t], want_w[t], rtol=1e-5, atol=1e-7)
        row = np.zeros(E)
        row[want_chosen[t]] = want_w[t]
        assert np.allclose(dense[t], row, rtol=1e-5, atol=1e-7)


@pytest.mark.parametrize("out", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,d,E,identity,top,ff", [(1, 64, 4, 2, 3, 16), (9, 50, 3, 5, 6, 9), (16, 72, 6, 1, 2, 24)])
def test_experts_that_give_their_input_back(T, d, E, identity, top, ff, out):
    """Both ways of a step: the chosen experts alone (few rows), whose indices behind the experts stand for the input, and
    all experts side by side with a mix that holds more numbers than there are experts."""
    from nanoinfer_amd import kernels as K
    dev = torch.device("cuda")
    g = torch.Generator().manual_seed(T + d)
    x = torch.randn(T, d, generator=g).to(out)
    up = (torch.randn(E * 2 * ff, d, generator=g) * 0.2).to(out)
    down = (torch.randn(d, E * ff, generator=g) * 0.2).to(out)
    chosen = torch.stack([torch.randperm(E + identity, generator=g)[:top] for _ in range(T)]).to(torch.int32)
    chosen[0, 0] = E                                   # at least one of them
    chosen[0, 1:] = torch.tensor([e for e in range(E + identity) if e != E][: top - 1], dtype=torch.int32)
    mix = torch.rand(T, top, generator=g)
    want = np.zeros((T, d))
    w = {}
    for e in range(E):
        w[f"e{e}.gate"], w[f"e{e}.up"] = up[e * 2 * ff:e * 2 * ff + ff].double().numpy(), up[e * 2 * ff + ff:(e + 1) * 2 * ff].double().numpy()
        w[f"e{e}.down"] = down[:, e * ff:(e + 1) * ff].double().numpy()
    xd = x.double().numpy()
    for t in range(T):
        for e, a in zip(chosen[t].tolist(), mix[t].double().tolist()):
            want[t] += a * (xd[t] if e >= E else P.expert(xd[t:t + 1], w, f"e{e}.", 1.5)[0])
    tol = 1e-5 if out == torch.float32 else 1e-2
    got = K.experts_few(x.to(dev), up.to(dev), down.to(dev), chosen.to(dev), mix.to(dev), ff, "capped_glu", limit=1.5, slope=1.702)
    assert float(np.abs(got.double().cpu().numpy() - want).max()) <= tol * np.abs(want).max()
    mix_all = torch.zeros(T, E + identity).scatter_(1, chosen.long(), mix).to(dev)
    act = K.experts_act(K.linear(x.to(dev), up.to(dev)), mix_all, ff, "capped_glu", 1.5, 1.702)
    total = K.linear(act, down.to(dev), out_dtype=torch.float32)
    total += K.identity_experts(x.to(dev), mix_all, E, torch.empty(T, d, dtype=torch.float32, device=dev))
    assert float(np.abs(total.double().cpu().numpy() - want).max()) <= (1e-5 if out == torch.float32 else 2e-2) * np.abs(want).max()


@pytest.mark.parametrize("out", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("M,N,Kd", [(1, 144, 64), (8, 40, 2048), (16, 33, 50), (17, 96, 128), (40, 2050, 64), (64, 160, 72), (200, 77, 96)])
def test_a_product_with_squared_relu(M, N, Kd, out):
    """``relu(x W^T)^2`` through the skinny product's own store and, for many rows or odd sizes, behind the library's."""
    from nanoinfer_amd import kernels as K
    dev = torch.device("cuda")
    g = torch.Generator().manual_seed(M + N)
    x, w = torch.randn(M, Kd, generator=g).to(out), (torch.randn(N, Kd, generator=g) * Kd ** -0.5).to(out)
    want = (x.double() @ w.double().T).clamp(min=0) ** 2
    for weight in (K.Weight(w.to(dev)), K.Weight(w.to(dev), tiled=False)):
        got = K.linear_relu2(x.to(dev), weight)
        assert got.dtype == out and float((got.double().cpu() - want).abs().max()) <= (1e-5 if out == torch.float32 else 1.6e-2) * float(want.max())


@pytest.mark.parametrize("table", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("d", [64, 37, 2])
def test_the_sinusoid_of_the_embedding(d, table):
    """A row of the table plus a sinusoid of the position, at positions up to a million: the angle is not rounded to
    float32 before it is brought near zero."""
    from nanoinfer_amd import kernels as K
    dev = torch.device("cuda")
    g = torch.Generator().manual_seed(d)
    E = torch.randn(20, d, generator=g).to(table)
    positions = torch.tensor([0, 1, 2, 63, 1023, 4097, 65537, 999983], dtype=torch.int32)
    ids = torch.tensor([3, 0, 19, 7, 7, 1, 2, 5], dtype=torch.int32)
    freq = torch.tensor([P.SINUSOID_BASE ** (-2.0 * i / d) for i in range((d + 1) // 2)], dtype=torch.float64)
    out = torch.empty(8, d, dtype=torch.float32, device=dev)
    K.embed_scaled(ids.to(dev), positions.to(dev), E.to(dev), None, 1.0, out, freq=freq.to(dev))
    want = E.double().numpy()[ids.numpy()] + P.sinusoid(positions.numpy(), d)
    assert float(np.abs(out.double().cpu().numpy() - want).max()) <= 1e-6


# ------------------------------------------------------------------ generation through the framework's entry points

@pytest.mark.parametrize("name", ["mixed", "shared_kv"])
def test_greedy_generation_through_the_engine_is_the_plain_greedy(name):
    """``Engine.generate`` (scheduler, chunked prompts, recorded decode runs, preemption on a pool that is too small)
    gives the tokens that the plain implementation's argmax gives, wherever the plain logits leave no doubt."""
    from nanoinfer_amd.engine.llm import Engine
    from nanoinfer_amd.engine.scheduler import EngineConfig
    from nanoinfer_amd.sampling.params import SamplingParams
    folder = folder_of(name)
    cfg, w = _model(folder)
    prompts = [list(random_tokens(cfg["vocab"], n, 300 + n)) for n in (3, 26, 11, 40, 1)]
    new = 20
    eng = Engine(folder, EngineConfig(dtype="float32", block_size=8, num_cache_blocks=10, max_sequences=3, admission_headroom=0,
                                      prefill_chunk_size=16, max_num_batched_tokens=40), ignore_eos=True)
    results = eng.generate(prompts, max_new_tokens=new, params=SamplingParams.greedy())
    assert eng.scheduler.num_preemptions > 0, "the pool was meant to be too small for all"
    checked = 0
    for prompt, res in zip(prompts, results):
        toks = list(prompt)
        assert len(res.tokens) == new
        for t in res.tokens:
            row = P.forward(cfg, w, toks)[-1]
            top = np.sort(row)[-2:]
            if float(top[1] - top[0]) > 1e-3 * float(np.abs(row).max()):
                assert t == int(row.argmax()), (len(prompt), len(toks))
                checked += 1
            toks.append(t)
    assert checked >= len(prompts) * new * 3 // 4
    eng.runner.cache.check()
    assert all_pages_free(eng.runner.cache)


def test_sampling_with_temperature_runs_and_respects_the_seed():
    from nanoinfer_amd.engine.llm import Engine
    from nanoinfer_amd.engine.scheduler import EngineConfig
    from nanoinfer_amd.sampling.params import SamplingParams
    folder = folder_of("mixed")
    prompts = [list(random_tokens(Z.MIXED["vocab"], n, 500 + n)) for n in (9, 20)]
    outs = []
    for _ in range(2):
        eng = Engine(folder, EngineConfig(dtype="bfloat16", block_size=8, num_cache_blocks=64, max_sequences=4), ignore_eos=True)
        outs.append([r.tokens for r in eng.generate(prompts, max_new_tokens=10,
                                                    params=SamplingParams(temperature=0.8, top_k=20, top_p=0.9, seed=5))])
    assert outs[0] == outs[1] and all(len(t) == 10 for t in outs[0])


def test_the_command_line_generates_from_a_fuvevik_folder(tmp_path, capsys):
    """``bin/nanoinfer``'s program with a Fuvevik ``config.json``: the random-weights mode writes the folder, the engine
    generates greedily from two prompts, and the tokens are the plain implementation's."""
    from nanoinfer_amd import cli
    cfg_path, folder = str(tmp_path / "config.json"), str(tmp_path / "model")
    with open(cfg_path, "w") as fh:
        json.dump(Z.SHARED_KV, fh)
    rc = cli.main(["--random-config", cfg_path, "--save-random-model", folder, "--random-seed", "3", "--dtype", "fp32",
                   "--prompt-ids", "5,9,77,3,90", "--prompt-len", "19", "--max-tokens", "6", "--ignore-eos", "--json",
                   "--num-cache-blocks", "32", "--block-size", "8"])
    assert rc == 0
    lines = [json.loads(l) for l in capsys.readouterr().out.splitlines() if l.startswith("{")]
    assert len(lines) == 2 and lines[0]["prompt_len"] == 5 and lines[1]["prompt_len"] == 19
    cfg, w = P.read_model_folder(folder)
    toks = [5, 9, 77, 3, 90]
    for t in lines[0]["tokens"]:
        row = P.forward(cfg, w, toks)[-1]
        top = np.sort(row)[-2:]
        if float(top[1] - top[0]) > 1e-3 * float(np.abs(row).max()):
            assert t == int(row.argmax())
        toks.append(t)


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_trace_program_replays_a_fuvevik_model(dtype, tmp_path):
    """``bin/trace_run`` in a process of its own, four slots: portions beside single tokens, a request that pauses, a
    fifth request on a slot and pages that another has given back."""
    import subprocess
    import sys
    name = "mixed"
    folder = folder_of(name)
    vocab = Z.ALL[name]["vocab"]
    lengths = {"a": 70, "b": 33, "c": 9, "d": 52, "e": 41}
    requests = {r: random_tokens(vocab, n, 800 + i) for i, (r, n) in enumerate(lengths.items())}
    plan = [{"a": 30, "b": 2}, {"a": 1, "b": 31, "c": 8, "d": 20}, {"a": 1, "c": 1, "d": 1}, {"a": 37, "d": 31},
            {"a": 1, "e": 40}, {"e": 1}]
    done = {r: 0 for r in requests}
    lines, wanted = [], []
    for i, counts in enumerate(plan):
        entries, ended = [], []
        for r, c in counts.items():
            entries.append({"id": r, "tokens": list(requests[r][done[r]:done[r] + c]), "want": list(range(c))})
            wanted.append((i, r, done[r], c))
            done[r] += c
            if done[r] == len(requests[r]):
                ended.append(r)
        lines.append(json.dumps({"step": i, "entries": entries, "end": ended}))
    out_dir = str(tmp_path / "out")
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", dtype,
                           "--out", out_dir, "--max-tokens", "192", "--page-size", "8"],
                          input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done ")] == [f"done {i}" for i in range(len(plan))]
    rows = {r: [None] * len(requests[r]) for r in requests}
    for i in range(len(plan)):
        data = np.fromfile(os.path.join(out_dir, f"{i}.f32"), dtype="<f4").reshape(-1, vocab)
        at = 0
        for step, r, first, c in wanted:
            if step == i:
                for j in range(c):
                    rows[r][first + j] = torch.from_numpy(data[at + j].copy())
                at += c
        assert at == data.shape[0]
    for r, toks in requests.items():
        assert_close(torch.stack(rows[r]), plain(folder, toks), dtype, f"trace program, request {r}")
