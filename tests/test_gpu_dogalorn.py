"""Dogalorn on the GPU against the plain oracle (float64): every mechanism
alone, any cut of the tokens, mixed batches, reused pages and slots, keys
that stand out at chunk, page and tile edges, states that reach back, long
decoding and the framework's generation paths.

Caches and states start filled with NaN, so reading a position or a state
that the sequence has not written fails the comparison.
"""

import json
import os
import subprocess
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import dogalorn_oracle as O
from dogalorn_cases import (config, default, dense, greedy, memory, needle,
                            only, pair, rel, save, ssd, tokens, weights, worst)
from dogalorn_oracle import Oracle
from layered_gpu import EXACT, ROUNDED, cut, engine, entry, run

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])


# ---------------------------------------------------------------- kernels

def _dev(a, dtype=torch.float32):
    return torch.from_numpy(np.asarray(a, np.float32)).to("cuda", dtype)


def _np(t):
    return t.double().cpu().numpy()


def _i32(v):
    return torch.tensor(v, dtype=torch.int32, device="cuda")


def _nan(*shape, dtype=torch.float32):
    return torch.full(shape, float("nan"), dtype=dtype, device="cuda")


@DTYPES
@pytest.mark.parametrize("S", [1, 2, 5])
@pytest.mark.parametrize("W", [8, 300, 1030])
def test_embedding_of_token_pairs(dtype, S, W):
    """Single tokens beside runs, at a sequence's start and later; products
    beyond 32 bits; the tokens left for the next step."""
    from llm_np_cp_amd.ops import hybrid_ops as hy

    rng = np.random.default_rng(W)
    V, buckets = 30000, 97
    spec = SimpleNamespace(mul_prev=91139, mul_cur=70001, buckets=buckets)
    table = torch.randn(V, W, device="cuda").to(dtype)
    pairs = torch.randn(buckets + 1, W, device="cuda").to(dtype)
    lens, slots, pos0 = [1, 1, 1, 2, 70, 3], [4, 0, 6, 1, 3, 5], [
        0, 5, 64, 0, 9, 1]
    ids = rng.integers(0, V, sum(lens))
    row0 = np.concatenate([[0], np.cumsum(lens)[:-1]])
    last = rng.integers(0, V, 7)
    b = SimpleNamespace(
        T=len(ids), nd=3, nseg=3, ids=_i32(ids.tolist()),
        slot=_i32(np.repeat(slots, lens).tolist()),
        pos=_i32([p + k for p, n in zip(pos0, lens) for k in range(n)]),
        seg_row0=_i32(row0.tolist()), seg_len=_i32(lens),
        seg_slot=_i32(slots))
    keep, x = _i32(last.tolist()), _nan(len(ids), S, W)
    hy.embed_pairs(table, pairs, keep, b, x, W, S, spec)
    w = {"embed": _np(table), "bigram": _np(pairs)}
    s = dict(buckets=buckets, mul_prev=91139, mul_cur=70001)
    left = last.copy()
    for r, n, q, p in zip(row0, lens, slots, pos0):
        want = O.embed(w, s, ids[r:r + n], last[q] if p else None)
        for k in range(S):
            assert rel(_np(x[r:r + n, k]), want) < 1e-6
        left[q] = ids[r + n - 1]
    assert keep.tolist() == left.tolist()


def _streams(S, W, n, halves, seed):
    rng = np.random.default_rng(seed)
    R = rng.standard_normal
    d = dict(x=R((n, S, W)), y=R((n, W)), mix=R((S, S)), feed=R(S), read=R(S),
             g=R(()) + 2)
    if halves:
        d.update(y2=3 * R((n, W)), gb=R(W), gb2=R(W))
    return d


def _turned(d, eps):
    y = d["y"]
    if "y2" in d:
        y = O.halves(y, d["y2"], d["gb"], d["gb2"], eps)
    xs = O.spread([d["x"][:, s] for s in range(d["x"].shape[1])], d["mix"],
                  d["feed"], y)
    return np.stack(xs, 1), O.rms(O.gather(xs, d["read"]), eps) * d["g"]


@DTYPES
@pytest.mark.parametrize("S", [1, 2, 3, 4, 8])
@pytest.mark.parametrize("W", [8, 88, 1029, 2048, 3000, 4100])
def test_streams_turn_and_are_read(dtype, S, W):
    from llm_np_cp_amd.ops import hybrid_ops as hy

    n, Kp, eps, N = 5, -(-W // 64) * 64, 1e-2, 37
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    M = torch.zeros(N, Kp, dtype=dtype, device="cuda")
    M[:, :W] = _dev(np.random.default_rng(1).standard_normal((N, W)) /
                    W ** .5, dtype)
    for halves in (False, True):
        d = _streams(S, W, n, halves, W + S)
        xs, h = _turned(d, eps)
        kw = {k: _dev(v) for k, v in d.items() if k != "x"}
        x = _dev(d["x"])
        for place in (x.clone(), _nan(n, S, W)):       # in place and beside
            src = place if not place.isnan().any() else x
            out = _nan(n, Kp, dtype=dtype)
            hy.hyper_rows(src, out, n, W, Kp, eps, S, xout=place, **kw)
            assert rel(_np(place), xs) < 1e-5
            assert rel(_np(out[:, :W]), h) < tol and (out[:, W:] == 0).all()
        # picked rows; nothing due; nothing read
        out = _nan(2, Kp, dtype=dtype)
        hy.hyper_rows(x, out, 2, W, Kp, eps, S, rows=_i32([4, 1]), **kw)
        assert rel(_np(out[:, :W]), h[[4, 1]]) < tol
        out = _nan(n, Kp, dtype=dtype)
        hy.hyper_rows(x, out, n, W, Kp, eps, S, read=kw["read"], g=kw["g"])
        plain = O.gather([d["x"][:, s] for s in range(S)], d["read"])
        assert rel(_np(out[:, :W]), O.rms(plain, eps) * d["g"]) < tol
        due = {k: v for k, v in kw.items() if k not in ("read", "g")}
        xo = x.clone()
        hy.hyper_rows(xo, None, n, W, W, eps, S, xout=xo, **due)
        assert rel(_np(xo), xs) < 1e-5
        # a single row inside a projection
        one = {k: v[2] if k in ("y", "y2") else v for k, v in kw.items()}
        y, xo = torch.full((N + 1,), 7.0, device="cuda"), _nan(S, W)
        hout = _nan(Kp, dtype=dtype)
        hy.lin_row(M, x[2], y, W, eps, hout=hout, hyper=dict(
            S=S, xout=xo, **one))
        assert rel(_np(xo), xs[2]) < 1e-5 and y[N] == 7.0
        assert rel(_np(hout[:W]), h[2]) < tol and (hout[W:] == 0).all()
        assert rel(_np(y[:N]), h[2] @ _np(M[:, :W]).T) < tol
        y[:] = 0
        hy.lin_row(M, x, y, W, eps, rows=_i32([3]), hyper=dict(S=S, **kw))
        assert rel(_np(y[:N]), h[3] @ _np(M[:, :W]).T) < tol


@DTYPES
@pytest.mark.parametrize("W, groups", [
    (8, 1), (8, 8), (120, 2), (192, 3), (2048, 1), (2048, 8), (3000, 5),
    (4096, 64), (6144, 1024)])
def test_norm_in_equal_parts(dtype, W, groups):
    from llm_np_cp_amd.ops import hybrid_ops as hy

    rng = np.random.default_rng(W)
    n, Kp, N, eps = 4, -(-W // 64) * 64, 29, 1e-2
    x = rng.standard_normal((n, W)) * np.repeat(
        rng.uniform(0.1, 5, groups), W // groups)
    g = 1 + 0.3 * rng.standard_normal(W)
    want = O.group_norm(x, g, groups, eps)
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    out = _nan(n, Kp, dtype=dtype)
    hy.group_rows(_dev(x), _dev(g), out, n, W, Kp, eps, groups)
    assert rel(_np(out[:, :W]), want) < tol and (out[:, W:] == 0).all()
    M = torch.zeros(N, Kp, dtype=dtype, device="cuda")
    M[:, :W] = _dev(rng.standard_normal((N, W)) / W ** .5, dtype)
    y = torch.full((N + 1,), 7.0, device="cuda")
    hy.lin_row(M, _dev(x[1]), y, W, eps, g=_dev(g), groups=groups)
    assert rel(_np(y[:N]), want[1] @ _np(M[:, :W]).T) < tol and y[N] == 7.0


@DTYPES
@pytest.mark.parametrize("M", [1, 2, 19, 40, 90, 300])
@pytest.mark.parametrize("K, K2", [(64, 192), (320, 64), (1024, 1152)])
def test_two_products_of_unequal_depth(dtype, M, K, K2):
    from llm_np_cp_amd.ops import hybrid_ops as hy

    g = torch.Generator(device="cuda").manual_seed(M)
    R = lambda *s: torch.randn(*s, device="cuda", generator=g).to(dtype)
    N, half = 77, M * 77 + 5
    X, W1, W2 = R(M, K + K2), R(N, K) / K ** .5, R(N, K2) / K2 ** .5
    W, Y = torch.cat([W1.flatten(), W2.flatten()]), _nan(2 * half)
    if M == 1:
        hy.lin_row(W[:N * K].view(N, K), None, Y, 0, 0.0, hin=X.flatten(),
                   second=(K2, K, N * K, half))
    else:
        hy.gemm_rows(X, W, Y, M, K + K2, N, hy.EPI_F32, N=N, K=K, Z=2, xz=K,
                     wz=N * K, yz=half, K2=K2)
    tol = 2e-5 if dtype == torch.float32 else 5e-3
    for at, a, w in ((0, X[:, :K], W1), (half, X[:, K:], W2)):
        got = _np(Y[at:at + M * N]).reshape(M, N)
        assert rel(got, _np(a) @ _np(w).T) < tol
    assert Y[M * N:half].isnan().all() and Y[half + M * N:].isnan().all()


@DTYPES
@pytest.mark.parametrize("M", [1, 3, 40, 200])
def test_gelu_with_bias(dtype, M):
    from llm_np_cp_amd.ops import hybrid_ops as hy

    rng = np.random.default_rng(M)
    N, K = 90, 128
    X, W = _dev(rng.standard_normal((M, K)), dtype), _dev(
        rng.standard_normal((N, K)) / 6, dtype)
    bias, Y = _dev(rng.standard_normal(N)), _nan(M, N, dtype=dtype)
    if M == 1:
        hy.lin_row(W, None, Y[0], 0, 0.0, hin=X[0], bias=bias, epi=hy.EPI_GELU)
    else:
        hy.gemm_rows(X, W, Y, M, K, N, hy.EPI_GELU, bias=bias)
    want = O.gelu(_np(X) @ _np(W).T + _np(bias))
    assert rel(_np(Y), want) < (1e-5 if dtype == torch.float32 else 5e-3)


def test_launchers_refuse_bad_shapes():
    from llm_np_cp_amd.ops import hybrid_ops as hy

    t = torch.zeros(64, 64, device="cuda")
    i = torch.zeros(64, dtype=torch.int32, device="cuda")
    bad = [
        lambda: hy.hyper_rows(t, t, 2, 64, 64, 1e-5, 9, read=t, g=t),
        lambda: hy.hyper_rows(t, t, 2, 64, 64, 1e-5, 2, read=t),
        lambda: hy.hyper_rows(t, t, 2, 64, 64, 1e-5, 2, read=t, g=t, y=t),
        lambda: hy.hyper_rows(t, t, 2, 64, 64, 1e-5, 2, read=t, g=t, rows=i,
                              xout=t),
        lambda: hy.lin_row(t, t, t[0], 64, 1e-5, hyper=dict(
            S=2, read=t, g=t, y=t, mix=t[:2, :2], feed=t, xout=t)),
        lambda: hy.group_rows(t, t, t, 2, 64, 64, 1e-5, 7),
        lambda: hy.lin_row(t, t, t[0], 64, 1e-5, g=t, groups=5),
        lambda: hy.lin_row(t, None, t, 0, 0.0, hin=t, second=(63, 64, 0, 64)),
        lambda: hy.gemm_rows(t, t, t, 2, 64, 64, hy.EPI_F32, N=2, Z=2, K2=65),
        lambda: hy.mingru_step(1, hy.MingruArgs().put(C=8, ldo=7, rows=1)),
        lambda: hy.mingru_run(1, hy.MingruArgs().put(C=8, ldo=8, nchunk=0)),
        lambda: hy.ssd_step(hy.SsdArgs().put(rows=1, H=4, G=3, N=8, vd=8,
                                             nvt=1, C=80, taps=4)),
        lambda: hy.ssd_run(hy.SsdArgs().put(rows=1, H=4, G=2, N=8, vd=8, nvt=1,
                                            C=63, taps=4, nseg=1, nchunk=1)),
        lambda: hy.gqa_token(1, hy.GqaArgs().put(
            rows=1, G=1, H=1, d=8, DP=64, vd=8, VP=64, ldo=8, NS=1, bias=t)),
    ]
    for k, f in enumerate(bad):
        with pytest.raises(RuntimeError):
            f()
            pytest.fail(f"case {k}")


# -------------------------------------------------------- mechanisms alone

def check_alone(cfg, n=150, seed=0, cuts=None, w=None, **kw):
    w, t = w or weights(cfg, seed, **kw), tokens(cfg, n)
    want, _ = Oracle(cfg, w).run(t)
    cuts = cuts or ([n], [1] * 70 + [2, n - 72], cut(n, [64, 1, 65, 20]))
    m = engine(cfg, w)
    for c in cuts:
        assert worst(run(m, t, c), want) < EXACT, c
    m = engine(cfg, w, "bf16")
    for c in cuts:
        assert rel(run(m, t, c), want) < ROUNDED, c


def one_half(p, half, seed, buckets=10):
    cfg = config([(p, None)])
    return cfg, only(cfg, weights(cfg, seed, buckets), half)


# heads, kv_heads, dim, chunk, far; rows of biases
ATTENTIONS = [(4, 2, 20, 45, 30, 10), (1, 1, 8, 1, 9, 2), (5, 1, 64, 64, 100, 16),
              (16, 2, 24, 63, 40, 32), (40, 2, 16, 65, 17, 12), (3, 3, 65, 7, 90, 6),
              (2, 1, 128, 128, 128, 32), (2, 2, 130, 100, 64, 24),
              (6, 3, 256, 129, 33, 4), (17, 1, 33, 4096, 50, 20),
              (8, 8, 64, 2, 3, 4), (4, 4, 96, 150, 149, 64)]


@pytest.mark.parametrize("k", range(len(ATTENTIONS)))
def test_chunked_attention_alone(k):
    *a, rows = ATTENTIONS[k]
    cfg, w = one_half(pair(*a, scale=0.31 if k % 2 else None), "left", k, rows)
    check_alone(cfg, w=w)


@pytest.mark.parametrize("width", [1, 40, 64, 92, 260, 1000])
def test_gated_recurrence_alone(width):
    cfg, w = one_half(pair(width=width), "right", width)
    check_alone(cfg, w=w)


@pytest.mark.parametrize("a", [
    dict(), dict(heads=1, vdim=1, state=1, groups=1, conv=1, norm_groups=1),
    dict(heads=4, vdim=64, state=64, groups=1, conv=4, norm_groups=4),
    dict(heads=3, vdim=65, state=130, groups=3, conv=2, norm_groups=5),
    dict(heads=8, vdim=16, state=128, groups=2, conv=3, norm_groups=8),
    dict(heads=2, vdim=130, state=16, groups=1, conv=7, norm_groups=1),
    dict(heads=5, vdim=36, state=70, groups=5, conv=5, norm_groups=3),
    dict(heads=4, vdim=12, state=300, groups=4, conv=12, norm_groups=16)])
def test_state_space_alone(a):
    check_alone(config([(ssd(**a), None)]), seed=a.get("state", 0))


@pytest.mark.parametrize("a", [
    dict(heads=64, vdim=8, groups=4), dict(heads=24, vdim=70, state=150)])
def test_state_space_decode_batches(a):
    """Few and many blocks in the step of single tokens, beside a run."""
    cfg = config([(ssd(**a), None)])
    w, t = weights(cfg), tokens(cfg, 60)
    want, _ = Oracle(cfg, w).run(t)
    m = engine(cfg, w, max_batch=17)
    seqs = [m.open_sequence() for _ in range(17)]
    m.step([entry(s, t[:2 * k + 1], []) for k, s in enumerate(seqs)])
    for n in range(4):
        got = m.step([entry(s, t[2 * k + 1 + n:][:1])
                      for k, s in enumerate(seqs)]).cpu().numpy()
        assert worst(got, want[1 + n:34 + n:2]) < EXACT
    got = m.step([entry(s, t[2 * k + 5:][:1 if k else 3])
                  for k, s in enumerate(seqs)]).cpu().numpy()
    assert worst(got, np.concatenate([want[5:8], want[7:38:2]])) < EXACT


@pytest.mark.parametrize("ff", [1, 40, 64, 200, 5000])
def test_dense_alone(ff):
    """A mixer that writes nothing."""
    cfg = config([(ssd(), dense(ff))], width=72)
    w = weights(cfg)
    w["l0.mix.o"] *= 0
    check_alone(cfg, 90, cuts=([90], [1] * 90, [23, 2, 65]), w=w)


@pytest.mark.parametrize("kw", [
    dict(width=64, vocab=64), dict(width=130), dict(eps=0.3), dict(vocab=1001),
    dict(width=520), dict(streams=1), dict(streams=2), dict(streams=4),
    dict(streams=8), dict(logit_scale=1.0), dict(logit_scale=7.5),
    dict(buckets=1), dict(buckets=5003, muls=(900001, 700001)),
    dict(muls=(2, 1)), dict(muls=(1, 1))])
def test_stack_constants(kw):
    cfg = config([(pair(), dense(50)), (ssd(), None), (ssd(2, groups=1), dense(64)),
                  (pair(), dense(50), 0)], **kw)
    w, t = weights(cfg), tokens(cfg, 41)
    want, _ = Oracle(cfg, w).run(t)
    m = engine(cfg, w)
    for c in ([41], [1] * 41, [2, 10, 2, 1, 26]):
        assert worst(run(m, t, c), want) < EXACT


def test_shared_tensors_keep_their_own_state():
    cfg = config([(pair(), dense(50)), (ssd(), None), (pair(), dense(50), 0),
                  (pair(), dense(50), 2), (ssd(), None, 1)])
    w, t = weights(cfg), tokens(cfg, 80)
    want, _ = Oracle(cfg, w).run(t)
    m = engine(cfg, w)
    assert len(m.caches) == 5 and len(m.layers) == 2
    assert len({m.caches[k][0][0].data_ptr() for k in (0, 2, 3)}) == 3
    assert m.caches[1][0].data_ptr() != m.caches[4][0].data_ptr()
    for c in ([80], [1] * 80, [30, 2, 48]):
        assert worst(run(m, t, c), want) < EXACT


# ------------------------------------------------------------- whole model

@pytest.fixture(scope="module")
def model():
    cfg = default()
    w = weights(cfg)
    t = tokens(cfg, 300)
    return cfg, w, t, Oracle(cfg, w).run(t)[0]


def test_residual_after_every_layer_run(model):
    cfg, w, t, _ = model
    trace = []
    logits, _ = Oracle(cfg, w).run(t[:30], trace=trace)
    m = engine(cfg, w)
    got, hidden = m.forward_full(t[:30], return_hidden_states=True)
    assert len(hidden) == len(trace) + 1
    for a, b in zip(hidden[1:], trace):
        assert worst(a, b) < EXACT
    assert worst(got, logits) < EXACT


@pytest.mark.parametrize("sizes", [[300], [1], [2], [3, 1], [5, 2, 1],
                                   [63, 65], [64], [100, 1, 1, 27],
                                   [17, 2, 2, 130]])
def test_any_cut_gives_the_same_logits(model, sizes):
    cfg, w, t, want = model
    m = engine(cfg, w)
    assert worst(run(m, t, cut(300, sizes)), want) < EXACT


def test_scratch_smaller_than_the_step(model):
    """A step beyond the scratch rows runs as several batches."""
    cfg, w, t, want = model
    m = engine(cfg, w, prefill_chunk=64)
    assert m.PC == 64
    assert worst(run(m, t), want) < EXACT
    a, b = m.open_sequence(), m.open_sequence()
    got = m.step([entry(a, t[:50]), entry(b, t[:70])]).cpu().numpy()
    assert worst(got, np.concatenate([want[:50], want[:70]])) < EXACT


def test_bf16_whole_model(model):
    cfg, w, t, want = model
    m = engine(cfg, w, "bf16")
    for sizes in ([300], [1], [2, 70, 1]):
        assert rel(run(m, t, cut(300, sizes)), want) < ROUNDED


def test_long_prompt_with_split_keys():
    """Later portions of a long prompt: key splits of runs and tokens inside
    chunks that are long, short or never end, and many recurrence chunks."""
    cfg = config([(pair(8, 2, 40, 1100, 700, 70), None), (ssd(), dense(40)),
                  (pair(4, 1, 64, 4096, 90, 40), None),
                  (pair(6, 6, 24, 300, 256, 90), None)])
    w, t = weights(cfg), tokens(cfg, 1500)
    want, _ = Oracle(cfg, w).run(t)
    m = engine(cfg, w, max_seq=1536)
    for cuts in ([1500], [1200, 2, 3, 1, 1, 293], [700, 33, 767]):
        assert worst(run(m, t, cuts), want) < EXACT, cuts
    b = engine(cfg, w, "bf16", max_seq=1536)
    assert rel(run(b, t, [1200, 2, 3, 1, 1, 293]), want) < ROUNDED


def test_mixed_batches_with_reuse(model):
    """Random schedules over four live requests in a pool that is smaller
    than their sum: every logit equals the request's own run."""
    cfg, w, _, _ = model
    o = Oracle(cfg, w)
    reqs = [tokens(cfg, n, 10 + i) for i, n in enumerate(
        [150, 3, 64, 97, 1, 130, 65, 40, 128, 2, 77])]
    want = [o.run(t)[0] for t in reqs]
    m = engine(cfg, w, max_seq=192, pool_tokens=64 * 8)
    rng = np.random.default_rng(5)
    todo, live, at, used = list(range(len(reqs))), {}, {}, set()
    while todo or live:
        while todo and len(live) < 4:
            r = todo[0]
            held = sum(-(-len(reqs[k]) // 64) for k in live)
            if held + -(-len(reqs[r]) // 64) > 8:
                break
            live[todo.pop(0)] = m.open_sequence()
            at[r] = 0
        step, refs = [], []
        for r in rng.permutation(list(live)):
            if len(live) > 1 and rng.random() < 0.2:
                continue                       # left out of this step
            left = len(reqs[r]) - at[r]
            n = min(left, int(rng.choice([1, 1, 2, 3, 17, 63, 64, 65])))
            step.append(entry(live[r], reqs[r][at[r]:at[r] + n]))
            refs.append(want[r][at[r]:at[r] + n])
            at[r] += n
        if not step:
            continue
        got = m.step(step).cpu().numpy()
        assert worst(got, np.concatenate(refs)) < EXACT
        for r in list(live):
            used |= {(r, p) for p in live[r].pages}
            if at[r] == len(reqs[r]):
                m.close_sequence(live.pop(r))
    pages = [p for _, p in used]
    assert len(pages) > len(set(pages))        # pages did change hands
    assert m.cache.free_pages == 8 and m.cache.free_slots == 4


@pytest.mark.parametrize("rows", [2, 3, 5, 9, 16, 19, 40])
def test_many_single_tokens_in_one_step(model, rows):
    """Decode batches of every size class, at unequal lengths."""
    cfg, w, t, want = model
    m = engine(cfg, w, max_batch=rows)
    seqs = [m.open_sequence() for _ in range(rows)]
    lens = [1 + (7 * i) % 90 for i in range(rows)]
    m.step([entry(s, t[:n], []) for s, n in zip(seqs, lens)])
    for k in range(3):
        got = m.step([entry(s, t[n + k:n + k + 1])
                      for s, n in zip(seqs, lens)]).cpu().numpy()
        assert worst(got, np.stack([want[n + k] for n in lens])) < EXACT


def test_wanted_places_and_order(model):
    cfg, w, t, want = model
    m = engine(cfg, w)
    a, b, c = (m.open_sequence() for _ in range(3))
    got = m.step([entry(a, t[:20], [19, 0, 7]), entry(b, t[:1], [0]),
                  entry(c, t[:33], [])]).cpu().numpy()
    assert worst(got, want[[19, 0, 7, 0]]) < EXACT
    assert m.step([entry(c, t[33:40], [])]).shape == (0, cfg["vocab"])
    # one wanted row out of several: the pending addition of that row
    got = m.step([entry(b, t[1:3], [1]), entry(c, t[40:42], [])])
    assert worst(got.cpu().numpy(), want[2:3]) < EXACT


# ----------------------------------------- keys and inputs that stand out

@pytest.mark.parametrize("total", [64, 65, 130, 257])
@pytest.mark.parametrize("at", [0, 1, 15, 16, 31, 32, 62, 63, 64, 127, 128])
def test_key_that_stands_out(at, total):
    if at >= total - 1:
        pytest.skip("beyond the prompt")
    cfg, w, t = needle(at, total, 300)
    o = Oracle(cfg, w)
    want, _ = o.run(t)
    gone = t.copy()
    gone[at] = 3
    assert worst(o.run(gone)[0][-1:], want[-1:]) > 0.1     # it does show
    m = engine(cfg, w)
    for cuts in ([total], [total - 1, 1], [total - 2, 2],
                 cut(total - 1, [50, 3]) + [1]):
        assert worst(run(m, t, cuts)[-1:], want[-1:]) < EXACT
    b = engine(cfg, w, "bf16")
    for cuts in ([total], [total - 1, 1]):
        assert rel(run(b, t, cuts)[-1:], want[-1:]) < ROUNDED


@pytest.mark.parametrize("chunk", [2, 3, 31, 32, 33, 63, 64, 65, 100, 128])
@pytest.mark.parametrize("heads", [(1, 1), (4, 2), (20, 1)])
def test_chunk_edges(chunk, heads):
    """The key that stands out is a chunk's first token or the one ahead of
    it; the asking token is the chunk's last or comes earlier."""
    for k in (1, 2, 256 // chunk):
        edge = k * chunk
        for at in (edge, edge - 1):
            for end in {edge + chunk - 1, edge + chunk // 2, edge + 1}:
                if end <= at or end < 4:
                    continue
                cfg, w, t = needle(at, end + 1, chunk, *heads)
                want = Oracle(cfg, w).run(t)[0][-1:]
                m = engine(cfg, w, max_seq=512)
                for cuts in ([end + 1], [end, 1], [end - 1, 2],
                             [at, end + 1 - at], [at + 1, end - at]):
                    cuts = [c for c in cuts if c]
                    assert worst(run(m, t, cuts)[-1:], want) < EXACT, (
                        at, end, cuts)


def test_chunk_edge_passes_over_decoded_tokens():
    """The asking token at every place while decoding: it sees the key until
    the chunk ends, and not one token longer."""
    cfg, w, t = needle(100, 200, 60, 3, 3)
    o = Oracle(cfg, w)
    m = engine(cfg, w)
    seqs = [m.open_sequence() for _ in range(2)]
    m.step([entry(s, t[:95], []) for s in seqs])
    _, st = o.run(t[:95])
    st0, shift = st, []
    for k in range(95, 150):
        z, st = o.run([1 if k == 100 else 2], st)
        z0, st0 = o.run([3 if k == 100 else 2], st0)     # without the key
        got = m.step([entry(seqs[0], [1 if k == 100 else 2])]).cpu().numpy()
        assert worst(got, z) < EXACT, k
        shift.append(np.abs(z - z0).max())
        # the second sequence goes on beside it, two tokens at a time
        if k % 2:
            m.step([entry(seqs[1], [2, 2], [])])
    assert min(shift[6:25]) > 0.05 and max(shift[25:]) < 1e-9   # ends at 120


@pytest.mark.parametrize("distance", [1, 4, 5, 6, 17, 29, 30, 31, 60, 100])
def test_distance_bias_of_one_bucket(distance):
    """One bucket stands out: the keys that are in it take the softmax."""
    rows, far = 10, 30
    cfg, w = one_half(pair(4, 2, 20, 128, far), "left", distance, rows)
    w["l0.mix.left.rel"] *= 0
    w["l0.mix.left.rel"][O.bucket(distance, rows, far)] = 9.0
    t = tokens(cfg, 125)
    want, _ = Oracle(cfg, w).run(t)
    flat = dict(w)
    flat["l0.mix.left.rel"] = w["l0.mix.left.rel"] * 0
    assert worst(Oracle(cfg, flat).run(t)[0][-1:], want[-1:]) > 0.05
    m = engine(cfg, w)
    for cuts in ([125], [1] * 125, [70, 2, 53]):
        assert worst(run(m, t, cuts), want) < EXACT


def test_sink_takes_weight_where_scores_are_low():
    """All scores far below the sink's 0, or far above it."""
    cfg, w = one_half(pair(5, 1, 20, 70, 30), "left", 4)
    t = tokens(cfg, 120)
    for bias in (-60.0, -4.0, 4.0, 60.0):
        w["l0.mix.left.rel"][:] = bias
        w["l0.mix.left.rel"][:, 2] = 0.5
        want, _ = Oracle(cfg, w).run(t)
        m = engine(cfg, w)
        for cuts in ([120], [1] * 120, [50, 2, 1, 67]):
            assert worst(run(m, t, cuts), want) < EXACT


@pytest.mark.parametrize("kind", ["mingru", "ssd"])
def test_state_reaches_back(kind):
    """The first token alone decides the last logits, through any cut; the
    slot's earlier sequence, with another first token, does not."""
    cfg, w, t = memory(kind, 200)
    other = t.copy()
    other[0] = 6
    o = Oracle(cfg, w)
    want, off = o.run(t)[0], o.run(other)[0]
    assert worst(off[-1:], want[-1:]) > 0.05
    m = engine(cfg, w, max_batch=1)
    for cuts in ([200], [1] * 200, [1, 199], [2] * 100, [64, 64, 72],
                 [63, 65, 72], [127, 1, 72], [198, 2]):
        run(m, other)
        assert worst(run(m, t, cuts), want) < EXACT, cuts


@pytest.mark.parametrize("taps", [1, 2, 3, 4, 6])
def test_convolution_window(taps):
    """With a state that forgets at once and the oldest tap as large as the
    rest, an input one place off or lost at a cut shows in the row that
    should see it last, and not in the next."""
    cfg = config([(ssd(conv=taps), None)])
    w, t = weights(cfg, 3), tokens(cfg, 80)
    w["bigram"] *= 0
    w["l0.mix.A_log"][:] = 8.0
    w["l0.mix.dt_bias"][:] = 2.0
    w["l0.mix.conv"][:, 0] = 1.0
    o = Oracle(cfg, w)
    want, _ = o.run(t)
    p = 40
    other = t.copy()
    other[p] = (t[p] + 7) % cfg["vocab"]
    off = o.run(other)[0]
    diff = np.abs(off - want).max(-1)
    assert diff[p + taps - 1] > 0.01 and diff[p + taps:].max() < 1e-6
    m = engine(cfg, w)
    for k in range(p, p + taps + 1):           # a cut at every place
        for cuts in ([k, 80 - k], [k] + [1] * (80 - k), [k, 2, 78 - k]):
            assert worst(run(m, t, cuts), want) < EXACT
            assert worst(run(m, other, cuts), off) < EXACT


def test_pair_across_every_cut():
    """The pair's earlier token lies in the step before, in another batch
    place or in the same portion; a sequence's first token has none."""
    cfg = config([(ssd(), None)], buckets=5003)
    w, t = weights(cfg), tokens(cfg, 40)
    w["bigram"] *= 3
    want, _ = Oracle(cfg, w).run(t)
    m = engine(cfg, w)
    for sizes in ([1], [2], [3, 1], [1, 2], [20]):
        assert worst(run(m, t, cut(40, sizes)), want) < EXACT
    a, b = m.open_sequence(), m.open_sequence()
    for k in range(0, 40, 4):                  # sequences side by side
        got = m.step([entry(b, t[k:k + 3]), entry(a, t[k:k + 1])])
        assert worst(got.cpu().numpy(), np.concatenate(
            [want[k:k + 3], want[k:k + 1]])) < EXACT
        got = m.step([entry(a, t[k + 1:k + 4]), entry(b, t[k + 3:k + 4])])
        assert worst(got.cpu().numpy(), np.concatenate(
            [want[k + 1:k + 4], want[k + 3:k + 4]])) < EXACT


def test_first_tokens_after_reuse(model):
    """A slot and pages that a long request left behind: one, two and three
    tokens alone, and the first tokens of a prompt, see none of it."""
    cfg, w, t, want = model
    m = engine(cfg, w, max_batch=1, max_seq=320, pool_tokens=320)
    for cuts in ([1], [2], [3], [1, 1, 1], [1, 2], [2, 1], [90]):
        run(m, t[100:300])
        n = sum(cuts)
        assert worst(run(m, t[:n], cuts), want[:n]) < EXACT


# ---------------------------------------------------- generation and serving

def test_long_greedy_decode_graph_and_eager(model):
    cfg, w, t, _ = model
    want, margin = greedy(cfg, w, t[:5], 180)
    assert margin > 1e-4
    m = engine(cfg, w)
    for graph in (True, False, True):
        m.prefill(t[:5])
        ids = m.decode(180, greedy=True, use_graph=graph)
        assert ids.tolist() == want
    assert m._graph_mode is not None and not getattr(m, "_graph_failed", 0)
    # chunks of the loop, and a token fed by hand afterwards
    m.prefill(t[:5])
    ids = np.concatenate([m.decode(n, greedy=True, first_from_logits=k == 0)
                          for k, n in enumerate([3, 16, 1, 60])])
    assert ids.tolist() == want[:80]


@pytest.mark.parametrize("B", [2, 4, 11])
def test_batched_generation(model, B):
    cfg, w, t, _ = model
    prompts = [t[i:i + 1 + 13 * i % 70] for i in range(B)]
    m = engine(cfg, w, max_batch=B)
    out = m.generate_tokens_batch(prompts, 40)
    for p, ids in zip(prompts, out):
        want, margin = greedy(cfg, w, p, 40)
        assert margin < 1e-4 or ids.tolist() == want


def test_rows_join_and_leave(model):
    """The server's row primitives: join, decode, retire, compact."""
    cfg, w, t, _ = model
    m = engine(cfg, w, max_batch=3)
    prompts = {0: t[:9], 1: t[20:85], 2: t[40:43], 3: t[:70]}
    want = {k: greedy(cfg, w, p, 20)[0] for k, p in prompts.items()}
    got = {}
    for k in (0, 1, 2):
        m.prefill_row(k, prompts[k])
        got[k] = [int(m.bt_next[k].item())]
    for k, ids in zip((0, 1, 2), m.decode_rows(3, 4)):
        got[k] += ids.tolist()
    m.compact_row(0, 2)                        # request 0 leaves
    assert m.rows[2] is None
    for k, ids in zip((2, 1), m.decode_rows(2, 5)):
        got[k] += ids.tolist()
    m.prefill_row(2, prompts[3])
    got[3] = [int(m.bt_next[2].item())]
    for k, ids in zip((2, 1, 3), m.decode_rows(3, 6)):
        got[k] += ids.tolist()
    for k in got:
        assert got[k] == want[k][:len(got[k])], k


def test_generate_session_and_rewind(tmp_path):
    import llm_np_cp_amd as L

    cfg = default(vocab=300)
    w = weights(cfg)
    save(cfg, w, tmp_path / "m")
    tok, m, c = L.load_model(str(tmp_path / "m"), dtype="fp32", max_seq=256)
    p = L.SamplingParams(strategy="greedy")
    prompt = "Once upon a time"
    ids = list(prompt.encode())
    want, _ = greedy(cfg, w, ids, 30)
    fast = L.generate(prompt, tok, m, max_tokens=30, params=p, stream=False)
    slow = L.generate(prompt, tok, m, max_tokens=30, params=p, stream=False,
                      logprobs=2)
    assert fast.token_ids == want and slow.token_ids == want
    assert len(L.generate(prompt, tok, m, max_tokens=12, params=L.
               SamplingParams(strategy="min_p", seed=1), stream=False,
               ).token_ids) == 12
    s = L.ChatSession(tok, m)
    a = s.send("Hi", max_tokens=6).token_ids
    b = s.send("more", max_tokens=6).token_ids
    hist = list(b"Hi")
    assert a == greedy(cfg, w, hist, 6)[0]
    assert b == greedy(cfg, w, hist + a + list(b"more"), 6)[0]
    m.prefill(np.asarray(ids))
    m.rewind(len(ids))
    with pytest.raises(ValueError, match="recurrent"):
        m.rewind(3)


def test_server_batches_requests(tmp_path):
    """The HTTP scheduler: concurrent greedy requests in one lockstep
    group give what each gives alone."""
    pytest.importorskip("fastapi")
    from concurrent.futures import ThreadPoolExecutor

    from fastapi.testclient import TestClient

    from llm_np_cp_amd.runtime.server import build_app

    cfg = config([(pair(), dense(60)), (ssd(), None), (pair(), dense(60), 0)],
                 vocab=280)
    w = weights(cfg)
    save(cfg, w, tmp_path / "m")
    app = build_app(str(tmp_path / "m"), backend="gpu", dtype="fp32",
                    max_seq=256, max_batch=3, batch_window_ms=60)
    prompts = ["a", "hello there", "x" * 70, "four", "The end."]
    want = [bytes(i % 256 for i in greedy(cfg, w, list(p.encode()), 12)[0])
            .decode("utf-8", errors="replace") for p in prompts]
    with TestClient(app) as c:
        def ask(p):
            return c.post("/v1/completions", json={
                "prompt": p, "max_tokens": 12, "strategy": "greedy",
                "stop_on_eos": False}).json()["choices"][0]["text"]
        with ThreadPoolExecutor(5) as ex:
            got = list(ex.map(ask, prompts))
        assert got == want
        assert c.get("/stats").json()["max_group"] > 1


def test_command_line(tmp_path):
    cfg = config([(pair(), dense(60)), (ssd(), dense())], vocab=300)
    w = weights(cfg)
    save(cfg, w, tmp_path / "m")
    p = subprocess.run(
        [sys.executable, "-m", "llm_np_cp_amd", "abc", "--model",
         str(tmp_path / "m"), "--backend", "gpu", "--dtype", "fp32",
         "--strategy", "greedy", "--max-tokens", "8"], cwd=ROOT,
        capture_output=True, timeout=100)
    assert p.returncode == 0, p.stderr.decode()[-2000:]
    want, _ = greedy(cfg, w, list(b"abc"), 8)
    text = bytes(i % 256 for i in want).decode("utf-8", errors="replace")
    assert text in p.stdout.decode("utf-8", errors="replace")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run(tmp_path, dtype):
    """The command: portions beside single tokens, slots given back and
    taken again, more requests over time than slots."""
    cfg = config([(pair(), dense()), (ssd(), None), (ssd(4, groups=2), dense(40)),
                  (pair(), dense(), 0)])
    w = weights(cfg)
    save(cfg, w, tmp_path / "m")
    (tmp_path / "out").mkdir()
    o = Oracle(cfg, w)
    reqs = {f"q{i}": tokens(cfg, n, i) for i, n in enumerate(
        [70, 5, 64, 2, 66, 30])}
    plan = [{"q0": 66, "q1": 2, "q2": 1}, {"q0": 1, "q1": 2, "q2": 60},
            {"q0": 1, "q3": 2, "q1": 1}, {"q2": 3, "q4": 65}, {"q0": 2},
            {"q4": 1, "q5": 29}, {"q5": 1}]
    at, lines, refs = dict.fromkeys(reqs, 0), [], []
    full = {k: o.run(t)[0] for k, t in reqs.items()}
    for n, step in enumerate(plan):
        entries, end, rows = [], [], []
        for k, c in step.items():
            lo, hi = at[k], at[k] + c
            want = [] if n == 3 else [c - 1] if c < 4 else [0, c - 1]
            entries.append({"id": k, "tokens": reqs[k][lo:hi].tolist(),
                            "want": want})
            rows += [full[k][lo + x] for x in want]
            at[k] = hi
            if hi == len(reqs[k]):
                end.append(k)
        lines.append(json.dumps({"step": n, "entries": entries, "end": end}))
        refs.append(rows)
    assert all(at[k] == len(reqs[k]) for k in reqs)
    p = subprocess.run(
        [os.path.join(ROOT, "bin", "trace_run"), "--model",
         str(tmp_path / "m"), "--dtype", dtype, "--out",
         str(tmp_path / "out"), "--max-tokens", "320"],
        input=("\n".join(lines) + "\n").encode(), capture_output=True,
        timeout=100)
    assert p.returncode == 0, p.stderr.decode()[-2000:]
    done = [l for l in p.stdout.decode().splitlines() if l.startswith("done")]
    assert done == [f"done {n}" for n in range(len(plan))]
    for n, rows in enumerate(refs):
        f = tmp_path / "out" / f"{n}.f32"
        assert f.exists() == bool(rows)
        if rows:
            got = np.fromfile(f, "<f4").reshape(-1, cfg["vocab"])
            if dtype == "float32":
                assert worst(got, np.stack(rows)) < EXACT
            else:
                assert rel(got, np.stack(rows)) < ROUNDED
