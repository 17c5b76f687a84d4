"""Fuvevik configurations drawn at random (the number of streams, head counts and groups, key and value sizes, score and
query factors, layers that read an earlier layer's keys and values, dense feed-forwards, experts, identity experts and how
many are chosen, limits, with and without each optional block of keys), each replayed in three ways in both compute types
against the plain implementation: the whole prompt, portions of changing size, and a prompt followed by single tokens."""
import os
import random
import shutil
import tempfile

import pytest

import fuvevik_configs as Z
from gpu_common import random_tokens
from test_gpu_fuvevik import assert_close, cuts, plain, replay, runner_for

pytestmark = pytest.mark.gpu


def draw(seed: int) -> dict:
    r = random.Random(seed)
    width = r.choice([32, 40, 50, 64, 72, 96, 128])
    layers, own = [], []           # own: (index, kv heads, dim, vdim) of layers that make their keys

    def feed_forward():
        kind = r.random()
        if kind < 0.2:
            return None
        if kind < 0.5:
            return Z.dense(r.choice([16, 37, 64, 160, 300]))
        experts = r.choice([1, 2, 5, 8, 12])
        identity = r.choice([None, 0, 1, 2, 4])
        shared = (r.choice([8, 24, 50]), r.choice([0.5, 1.0, 7.0])) if r.random() < 0.7 else None
        return Z.moe(experts, r.randint(1, min(6, experts + (identity or 0))), r.choice([8, 16, 20, 33]), r.choice([0.5, 1.5, 7.0]),
                     identity=identity, shared=shared)

    for i in range(r.randint(1, 6)):
        source = r.choice(own) if own and r.random() < 0.45 else None
        if source is None:
            kv, dim = r.choice([1, 2, 3, 4]), r.choice([8, 16, 20, 24, 32, 48, 64])
            vdim = r.choice([dim, 8, 16, 24, 80])
            own.append((i, kv, dim, vdim))
        else:
            _, kv, dim, vdim = source
        temp = (r.choice([0.1, 0.5, 1.0]), r.choice([1, 7, 16, 64, 200])) if r.random() < 0.8 else None
        layers.append((Z.attn(kv * r.choice([1, 2, 3, 5, 8]), kv, dim, vdim, r.choice([0.1, 0.25, 0.5]), temp=temp,
                              kv_from=source[0] if source else None), feed_forward()))
    return Z.model(width, r.choice([33, 64, 100, 257]), r.choice([1, 2, 2, 3, 4, 4, 5, 6, 8, 9]), layers, eps=r.choice([1e-6, 1e-5]))


_root = []


def folder_for(cfg, seed):
    import nanoinfer_amd  # noqa: F401
    from nanoinfer_amd.weights.loader import make_random_model
    if not _root:
        _root.append(tempfile.mkdtemp(prefix="fuvevik-random-"))
        import atexit
        atexit.register(shutil.rmtree, _root[0], ignore_errors=True)
    return make_random_model(os.path.join(_root[0], f"m{seed}"), cfg, seed, dtype="bfloat16", matrix_std=0.1)


@pytest.mark.parametrize("seed", list(range(1, 15)))
def test_a_configuration_drawn_at_random(seed):
    cfg = draw(seed)
    folder = folder_for(cfg, seed)
    toks = random_tokens(cfg["vocab"], 230 if seed % 3 == 0 else 90, seed)
    want = plain(folder, toks)
    rng = random.Random(seed)
    for dtype in ("float32", "bfloat16"):
        runner = runner_for(folder, dtype, page_size=rng.choice([1, 4, 8, 16, 32]))
        got = replay(runner, {"w": toks}, [{"w": len(toks)}])["w"]
        assert_close(got, want, dtype, f"seed {seed}: whole")
        sizes = [rng.choice([1, 2, 3, 5, 16, 31, 64]) for _ in range(5)]
        got = replay(runner, {"p": toks}, [{"p": c} for c in cuts(len(toks), sizes)])["p"]
        assert_close(got, want, dtype, f"seed {seed}: portions of {sizes}")
        first = rng.randint(1, len(toks) - 20)
        got = replay(runner, {"d": toks}, [{"d": first}] + [{"d": 1}] * (len(toks) - first))["d"]
        assert_close(got, want, dtype, f"seed {seed}: {first} tokens, then one by one")
        assert not runner.cache.live_requests()
