"""Nubedra models through the framework's engine against the plain oracle: prefill, decoding through the cache, portions,
used-again caches, several requests at once, recorded graphs, greedy generation, and the trace runner."""
import json
import os
import subprocess
from pathlib import Path

import numpy as np
import pytest

import nubedra_ref as ref
from folder_cases import MODES, Case, backend, done, engine, feed, held
from nubedra_util import CONFIGS, weights
from serisun_util import logit_error, write

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    return {k: Case(ref, tmp_path_factory.mktemp("nubedra") / k, c, weights(k, i)) for i, (k, c) in enumerate(CONFIGS.items())}


@pytest.fixture(params=sorted(MODES))
def be(request):
    b = backend(request.param)
    yield b
    done(b)


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("n", [1, 2, 7, 16, 17, 64, 65, 129, 200])
def test_a_whole_prompt(cases, be, name, n):
    c = cases[name]
    e = engine(c, be, n)
    t = c.tokens(n)
    held(feed(e, t, [n]), c.logits(t), be)
    e.close()


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_residual_stream_after_every_layer(cases, be, name):
    """Layer by layer: the first one that differs is the faulty one."""
    c = cases[name]
    t = c.tokens(30, 4)
    want = []
    ref.forward(t, c.cfg, c.w, want)
    for n in (30, 9, 1):
        got = []
        e = engine(c, be, 40)
        e.set_trace(lambda what, i, v: got.append((i, v.reshape(n, -1))) if what == "post_layer" else None)
        e.forward(t[:n])
        e.close()
        assert [i for i, _ in got] == list(range(len(want)))
        for (i, v), w in zip(got, want):
            d = np.sqrt(((v - w[:n]) ** 2).mean() / (w[:n] ** 2).mean())
            assert d < be.limit, f"layer {i}: {d:.2e}"


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("sizes", [[1], [2], [3, 2, 2, 11], [16, 1, 17, 64, 2], [63, 2, 1], [64, 64, 1], [65, 2], [8, 1, 1, 24, 32, 2], [150, 1]])
def test_portions_of_any_size(cases, be, name, sizes):
    """The logits at a position do not depend on how the prompt was cut: single tokens, pairs, and cuts just before, at and
    just after a tile's, a window's and a chunk's edge."""
    c = cases[name]
    t = c.tokens(170, 1)
    e = engine(c, be, 170)
    held(feed(e, t, sizes), c.logits(t), be, str(sizes))
    e.close()


def test_a_prompt_longer_than_the_engine_batch(cases, be):
    c = cases["mixed"]
    t = c.tokens(100, 2)
    e = engine(c, be, 128, max_batch=24)
    held(feed(e, t, [100]), c.logits(t), be)
    assert e.pos == 100
    e.reset()
    held(e.prefill(t)[None], c.logits(t)[-1:], be)
    e.close()


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_a_cache_that_is_used_again(cases, be, name):
    """Requests of unequal lengths one after the other on one engine: nothing of the last one is left."""
    c = cases[name]
    e = engine(c, be, 150)
    for k, n in enumerate((150, 3, 80, 1, 40)):
        t = c.tokens(n, 10 + k)
        e.reset()
        held(feed(e, t, [max(1, n // 2), 1, 2]), c.logits(t), be, f"request {k}")
    e.close()


def test_requests_that_take_turns(cases, be):
    """Three requests of unequal lengths on engines of their own over one backend, portions interleaved; one ends and its
    engine serves another meanwhile."""
    c = cases["mixed"]
    es = [engine(c, be, 90) for _ in range(3)]
    ts = [c.tokens(n, 20 + n) for n in (90, 31, 64)]
    at, got = [0, 0, 0], [[], [], []]
    r = np.random.default_rng(0)
    again = False
    while any(a < len(t) for a, t in zip(at, ts)):
        for k in range(3):
            n = min(int(r.choice([1, 1, 2, 5, 20])), len(ts[k]) - at[k])
            if n:
                got[k].append(es[k].forward_rows(ts[k][at[k]:at[k] + n], np.arange(n)))
                at[k] += n
        if at[1] == len(ts[1]) and not again:
            again = True
            held(np.concatenate(got[1]), c.logits(ts[1]), be)
            es[1].reset()
            ts[1], at[1], got[1] = c.tokens(50, 99), 0, []
    for k in range(3):
        held(np.concatenate(got[k]), c.logits(ts[k]), be, f"request {k}")
    for e in es:
        e.close()


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_long_decoding_from_recorded_graphs(cases, name):
    """Hundreds of single-token passes, most of them replays of one recorded graph, checked against the whole sequence; eager
    work (a portion, a checkpoint) in between; every pass equal to the eager backend's.  The windows pass over decoded tokens."""
    import inferred_hip as ih
    c = cases[name]
    t = c.tokens(330, 3)
    want = c.logits(t)
    runs = {}
    for graph in (True, False):
        b = ih.Hip(graph=graph)
        b.limit = 2e-2
        e = engine(c, b, 330)
        got = [feed(e, t[:20], [20])]
        for p in range(20, 330):
            if p in (150, 151):
                e.checkpoint()
            if p in (200, 201, 202):
                continue
            if p == 203:
                got.append(e.forward_rows(t[200:204], np.arange(4)))
                continue
            got.append(e.forward_rows(t[p:p + 1], [0]))
        runs[graph] = np.concatenate(got)
        s = b.graph_stats()
        assert b.take_error() is None
        assert (s["replays"] > 250 and s["captures"] >= 1) if graph else s["captures"] == 0
        e.close()
        held(runs[graph], want, b)
        b.close()
    assert np.array_equal(runs[True], runs[False])


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_greedy_generation(cases, name):
    """The framework's own generation, with ids chosen on the host (generate) and fed back on the device (decode_greedy), against
    the oracle's arg-max, token by token as long as its choice is clear."""
    import inferred_hip as ih
    c = cases[name]
    t = [int(x) for x in c.tokens(23, 7)]
    for kw in (dict(f32=True), {}):
        b = ih.Hip(**kw)
        e = engine(c, b, 80, max_batch=16)
        ids, _ = e.generate(t, 40)
        e.reset()
        e.prefill(t)
        dev = e.decode_greedy(40)
        e.close()
        assert b.take_error() is None
        b.close()
        assert len(ids) == 40 and list(ids) == list(dev)
        # (one pass over the oracle: a causal model's logits after every generated token)
        y = ref.forward(t + [int(i) for i in ids], c.cfg, c.w)[len(t) - 1:]
        lim, seen = 1e-4 if kw else 2e-2, 0
        for i, row in zip(ids, y):
            top = np.sort(row)[-2:]
            if top[1] - top[0] < 8 * lim * row.std():
                break
            assert int(i) == int(row.argmax())
            seen += 1
        assert seen > (10 if kw else 0)


def test_checkpoint_and_restore(cases, be):
    c = cases["mixed"]
    t = c.tokens(60, 8)
    e = engine(c, be, 60)
    feed(e, t[:25], [25])
    ck = e.checkpoint()
    first = feed(e, t[25:], [9, 1, 2])
    e.restore(ck)
    assert e.pos == 25 and not e.rewind(3)
    again = feed(e, t[25:], [9, 1, 2])
    assert np.array_equal(first, again)
    held(again, c.logits(t)[25:], be)
    e.close()


def test_a_model_without_recurrent_layers_can_be_rewound(cases, be):
    c = cases["windows"]
    t, u = c.tokens(90, 8), c.tokens(40, 9)
    e = engine(c, be, 120)
    feed(e, t, [40, 1, 2])
    assert e.rewind(70)
    held(feed(e, u, [20, 1, 2]), c.logits(np.concatenate([t[:70], u]))[70:], be)
    e.close()


def test_other_tensor_types_and_errors(cases, be, tmp_path):
    """Matrices in f32 and f16 beside bf16 ones; tokens and positions that are refused."""
    import inferred_hip as ih
    c = cases["odd"]
    d = write(tmp_path / "n", c.cfg, c.w, {"l0.mix.q": "F32", "l0.mix.a2": "F32", "l3.mix.a2": "F16", "embed": "F32", "l1.mix.uk": "F16", "l2.mix.uv": "F32",
                                           "l2.mix.uq": "F16", "l2.mlp.down": "F32", "l4.norm1b": "F16", "l1.mix.o": "F16"})
    m = ih.Model(d)
    t = c.tokens(70, 1)
    e = ih.Engine(m, be, 70)
    held(feed(e, t, [40, 1, 3, 20]), c.logits(t), be)
    with pytest.raises(ih.HipError, match="context overflow"):
        e.forward([1])
    e.reset()
    with pytest.raises(ih.HipError, match="outside the vocabulary"):
        e.forward([c.cfg["vocab"]])
    e.close()
    m.close()


# ---------------------------------------------------------------- the trace runner
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_the_trace_runner(cases, tmp_path, dtype):
    c = cases["mixed"]
    reqs = {"a": c.tokens(50, 1), "b": c.tokens(3, 2), "c": c.tokens(20, 3)}
    steps, at = [], {k: 0 for k in reqs}
    for name, n in [("a", 30), ("a", 1), ("a", 19), ("b", 3), ("c", 2), ("c", 18)]:
        lo = at[name]
        at[name] += n
        want = [] if (name, n) == ("c", 2) else [n - 1] if n < 3 else [2, 0, n - 1]   # in any order
        steps.append({"step": len(steps), "entries": [{"id": name, "tokens": [int(x) for x in reqs[name][lo:lo + n]], "want": want}],
                      "end": [name] if at[name] == len(reqs[name]) else []})
    env = {k: v for k, v in os.environ.items() if k != "HOME"}
    p = subprocess.run([str(ROOT / "bin" / "trace_run"), "--model", str(c.path), "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "50"],
                       input="".join(json.dumps(s) + "\n" for s in steps), stdout=subprocess.PIPE, stderr=subprocess.PIPE, text=True, timeout=90, env=env)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [x for x in p.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(len(steps))]
    lo = {k: 0 for k in reqs}
    for s in steps:
        x = s["entries"][0]
        f = tmp_path / f"{s['step']}.f32"
        if x["want"]:
            got = np.fromfile(f, "<f4").reshape(len(x["want"]), c.cfg["vocab"])
            want = c.logits(reqs[x["id"]])[[lo[x["id"]] + k for k in x["want"]]]
            assert logit_error(got, want).max() < (1e-4 if dtype == "float32" else 4e-2)
        else:
            assert not f.exists()
        lo[x["id"]] += len(x["tokens"])
