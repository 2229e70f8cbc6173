"""Fidizen on the GPU against the plain oracle (float64): every mechanism
alone, any cut of the tokens, mixed batches, reused pages and slots, keys
that stand out at window, page and tile edges, long decoding and the
framework's generation paths.

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

import fidizen_oracle as O
from fidizen_cases import (config, default, dense, greedy, latent, moe,
                           needle, rel, save, tokens, weights, worst)
from fidizen_oracle import Oracle
from layered_gpu import EXACT, ROUNDED, cut, engine, entry, run

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ---------------------------------------------------------------- kernels

def _dev(a, dtype=torch.float32):
    return torch.from_numpy(np.asarray(a, np.float32)).to("cuda", dtype)


def _np(t):
    return t.double().cpu().numpy()


def _batch(nd, runs, slots, pos):
    """Rows of nd single tokens and runs of the given lengths; sequence k
    has slots[k] and continues at pos[k]."""
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device="cuda")
    lens = [1] * nd + runs
    row0 = np.concatenate([[0], np.cumsum(lens)[:-1]]).tolist()
    chunks = [(row0[nd + g] + c, min(64, n - c), g)
              for g, n in enumerate(runs) for c in range(0, n, 64)]
    cols = list(zip(*chunks)) if chunks else [[0], [0], [0]]
    return SimpleNamespace(
        T=sum(lens), nd=nd, nseg=len(runs), nchunk=len(chunks),
        slot=i32(np.repeat(slots, lens).tolist()),
        pos=i32([p + k for p, n in zip(pos, lens) for k in range(n)]),
        seg_row0=i32(row0), seg_len=i32(lens), seg_slot=i32(slots),
        seg_pos0=i32(pos), chunk_row0=i32(cols[0]), chunk_len=i32(cols[1]),
        chunk_seg=i32(cols[2]))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 9, 13])
@pytest.mark.parametrize("width", [40, 66, 1029, 2048, 3000, 4096, 4100])
def test_input_convolution_of_rows(dtype, taps, width):
    """Post norm + addition + convolution, single tokens beside runs, at
    the start of a sequence and later, and the inputs left for later."""
    from llm_np_cp_amd.ops import hybrid_ops as hy

    rng = np.random.default_rng(width + taps)
    W, Kp, eps = width, -(-width // 64) * 64, 1e-4
    b = _batch(3, [2, 70, 9, 64], [5, 0, 3, 6, 1, 2, 4],
               [0, 1, 50, 0, 33, 64, 2])
    n, cw = b.T, rng.standard_normal((taps, W))
    x, y = 2 * rng.standard_normal((n, W)), rng.standard_normal((n, W))
    gb = 1 + 0.3 * rng.standard_normal(W)
    past = rng.standard_normal((7, taps, W))      # entry p % taps of a slot
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    for post in (False, True):
        v = x + O.rms(y, eps) * gb if post else x
        ring = _dev(past)
        for s in (5, 6):                          # sequences that start here
            ring[s] = float("nan")
        ring[0, 1 % taps:] = float("nan")         # position 0 only
        out = torch.full((n, Kp), float("nan"), dtype=dtype, device="cuda")
        xout = torch.full((n, W), float("nan"), device="cuda")
        kw = dict(y=_dev(y), gb=_dev(gb), xout=xout) if post else {}
        hy.conv_rows(_dev(x), out, b, W, Kp, eps, (
            _dev(cw), ring, b.slot, b.pos), **kw)
        if post:
            assert rel(_np(xout), v) < 1e-5
        assert (out[:, W:] == 0).all()
        got, left = _np(out[:, :W]), _np(ring)
        for r0, m, s, p0 in zip(*(t.tolist() for t in (
                b.seg_row0, b.seg_len, b.seg_slot, b.seg_pos0))):
            before = np.zeros((taps - 1, W))
            for j in range(1, min(taps - 1, p0) + 1):
                before[-j] = past[s, (p0 - j) % taps]
            want, _ = O.short_conv(v[r0:r0 + m], cw.T, before)
            assert rel(got[r0:r0 + m], want) < tol
            for j in range(1, min(taps, m + 1)):
                assert rel(left[s, (p0 + m - j) % taps], v[r0 + m - j]) < 1e-5


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("taps", [1, 2, 4, 7])
@pytest.mark.parametrize("width", [8, 88, 2048, 2113, 5000])
def test_one_row_projection_of_the_convolution(dtype, taps, width):
    from llm_np_cp_amd.ops import hybrid_ops as hy

    rng = np.random.default_rng(width)
    W, Kp, N, eps = width, -(-width // 64) * 64, 53, 1e-5
    x, y, past = (rng.standard_normal(s) for s in ((1, W), (1, W),
                                                   (taps, W)))
    gb, cw = 1 + rng.standard_normal(W), rng.standard_normal((taps, W))
    M = torch.zeros(N, Kp, dtype=dtype, device="cuda")
    M[:, :W] = _dev(rng.standard_normal((N, W)) / W ** .5, dtype)
    slot = torch.tensor([1], dtype=torch.int32, device="cuda")
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    v = x + O.rms(y, eps) * gb
    for p in (0, 1, 3, 100):
        pos = torch.tensor([p], dtype=torch.int32, device="cuda")
        before = np.zeros((taps - 1, W))
        ring = torch.full((2, taps, W), float("nan"), device="cuda")
        for j in range(1, min(taps - 1, p) + 1):
            before[-j] = past[j]
            ring[1, (p - j) % taps] = _dev(past[j])
        h, _ = O.short_conv(v, cw.T, before)
        got = torch.full((N + 1,), 7.0, device="cuda")
        xout = torch.full((W + 1,), 9.0, device="cuda")
        hout = torch.full((Kp,), float("nan"), dtype=dtype, device="cuda")
        hy.lin_row(M, _dev(x), got, W, eps, res=_dev(y), gb=_dev(gb),
                   conv=(_dev(cw), ring, slot, pos), hout=hout, xout=xout)
        assert rel(_np(got[:N]), h[0] @ _np(M[:, :W]).T) < tol
        assert got[N] == 7.0 and xout[W] == 9.0
        assert rel(_np(xout[:W]), v[0]) < 1e-5
        assert rel(_np(hout[:W]), h[0]) < tol and (hout[W:] == 0).all()
        assert rel(_np(ring[1, p % taps]), v[0]) < 1e-5


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("ff", [1, 40, 300, 4096, 9000, 11000])
def test_polynomial_activation(dtype, ff):
    from llm_np_cp_amd.ops import hybrid_ops as hy

    rng = np.random.default_rng(ff)
    n, Kp, N, eps = 3, -(-ff // 64) * 64, 37, 1e-3
    z = rng.standard_normal((n, ff)) * [[0.01], [1], [9]]
    coef = np.array([0.7, -1.1, 0.4, 0.25])
    tol = 2e-5 if dtype == torch.float32 else 1e-2
    Z = torch.full((n, Kp + 3), float("nan"), device="cuda")
    Z[:, :ff] = _dev(z)
    want = O.polynorm(z, coef, eps)
    out = torch.full((n, Kp), float("nan"), dtype=dtype, device="cuda")
    hy.poly_rows(Z, Kp + 3, _dev(coef), out, n, ff, eps)
    assert worst(_np(out[:, :ff]), want) < tol and (out[:, ff:] == 0).all()
    M = torch.zeros(N, Kp, dtype=dtype, device="cuda")
    M[:, :ff] = _dev(rng.standard_normal((N, ff)) / ff ** .5, dtype)
    y = torch.full((N + 1,), 7.0, device="cuda")
    for r in range(n):
        hy.lin_row(M, Z[r], y, ff, eps, act=_dev(coef))
        assert rel(_np(y[:N]), want[r] @ _np(M[:, :ff]).T) < tol
    assert y[N] == 7.0


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("M", [2, 17, 40, 70, 200, 1500])
def test_gemm_splits_and_rotates_queries(dtype, M):
    from llm_np_cp_amd.ops import hybrid_ops as hy

    g = torch.Generator(device="cuda").manual_seed(M)
    R = lambda *s: torch.randn(*s, device="cuda", generator=g)
    H, dp, RT, dims, K, CS = 3, 64, 32, 20, 128, 97
    N = H * (dp + RT)
    X, Wt = R(M, K).to(dtype), (R(N, K) / K ** 0.5).to(dtype)
    pos = torch.randint(0, 500, (M,), generator=g, device="cuda",
                        dtype=torch.int32)
    f = 1e4 ** (-2.0 * np.arange(dims // 2) / dims)
    ang = np.outer(np.arange(500), f)
    cos, sin = _dev(np.cos(ang)), _dev(np.sin(ang))
    qn = torch.full((M, H * dp), 5.0, dtype=dtype, device="cuda")
    qa = torch.full((M, H, CS), 5.0, dtype=dtype, device="cuda")
    rot = hy.Rotary().put(pos=pos, cosT=cos, sinT=sin,
                          y=qa.view(-1)[CS - RT:], split=H * dp, RT=RT,
                          dims=dims, ld=H * CS, hs=CS)
    hy.gemm_rows(X, Wt, qn, M, K, H * dp, hy.EPI_ROTARY, rotary=rot)
    ref = _np(X) @ _np(Wt).T
    tol = 2e-5 if dtype == torch.float32 else 5e-3
    assert rel(_np(qn), ref[:, :H * dp]) < tol
    want = O.rotate(ref[:, H * dp:].reshape(M, H, RT), _np(pos), 1e4, dims)
    assert rel(_np(qa[:, :, CS - RT:]), want) < tol
    assert (qa[:, :, :CS - RT] == 5.0).all()


@pytest.mark.parametrize("M", [3, 40, 90])
def test_gemm_gate_per_element(M):
    from llm_np_cp_amd.ops import hybrid_ops as hy

    g = torch.Generator(device="cuda").manual_seed(M)
    R = lambda *s: torch.randn(*s, device="cuda", generator=g)
    Z, N, K, ldo, ldg = 3, 28, 64, 128, 100
    X, Wt, gate = R(M, Z * K), R(Z, N, K), R(M, ldg)
    Y = torch.full((M, ldo), 5.0, device="cuda")
    hy.gemm_rows(X, Wt, Y, M, Z * K, ldo, hy.EPI_TGATE, N=N, K=K, Z=Z, xz=K,
                 wz=N * K, yz=N, gate=gate, ldg=ldg, gz=N, gc=1)
    ref = np.einsum("mzk,znk->mzn", _np(X).reshape(M, Z, K), _np(Wt))
    ref = ref.reshape(M, Z * N) / (1 + np.exp(-_np(gate)[:, :Z * N]))
    assert rel(_np(Y[:, :Z * N]), ref) < 1e-5 and (Y[:, Z * N:] == 5.0).all()


def test_launchers_refuse_bad_shapes():
    from llm_np_cp_amd.ops import hybrid_ops as hy

    t = torch.zeros(64, 64, device="cuda")
    i = torch.zeros(64, dtype=torch.int32, device="cuda")
    b = _batch(2, [], [0, 1], [0, 0])
    conv = (t[:3], torch.zeros(2, 3, 64, device="cuda"), i, i)
    with pytest.raises(RuntimeError):             # in place
        hy.conv_rows(t, t.clone(), b, 64, 64, 1e-5, conv, y=t, gb=t, xout=t)
    with pytest.raises(RuntimeError):             # a post norm needs xout
        hy.lin_row(t, t, torch.zeros(64, device="cuda"), 64, 1e-5, conv=conv,
                   res=t, gb=t)
    with pytest.raises(RuntimeError):             # queries without a latent
        hy.latent_mid(1, hy.LatentArgs().put(rows=1, H=1, RT=32, rot=2, RP=64,
                                             rank=9, dp=64, d=8, NS=1))
    with pytest.raises(RuntimeError):             # one choice too many
        m = hy.MoeArgs().put(idx=i, wt=t, ldh=64, ldact=64, W=64, E=2, K1=3,
                             ff=64, ffs=64)
        hy.moe_gu_few(1, m, hy.RouteArgs().put(z=t, idx=i, wt=t, ldz=2,
                                               lde=1, rows=1, E=2, top=3))
    with pytest.raises(RuntimeError):
        hy.gemm_rows(t, t, t, 2, 64, 64, hy.EPI_ROTARY, rotary=hy.Rotary().put(
            split=33, RT=31, dims=2))


# -------------------------------------------------------- mechanisms alone

def check_alone(cfg, n=150, seed=0, cuts=None, w=None):
    w, t = w or weights(cfg, seed), tokens(cfg, n)
    want, _ = Oracle(cfg, w).run(t)
    cuts = cuts or ([n], [1] * 70 + [2, n - 72], cut(n, [64, 1, 65, 20]))
    m = engine(cfg, w)
    for c in cuts:
        assert worst(run(m, t, c), want) < EXACT, c
    m = engine(cfg, w, "bf16")
    for c in cuts:
        assert rel(run(m, t, c), want) < ROUNDED, c


LATENTS = [latent(), latent(1, 8, 2, 1, 16, 8, 1), latent(window=2),
           latent(4, 32, 16, 32, 64, 64, 64), latent(5, 12, 8, 16, 70, 130, 33),
           latent(8, 64, 32, 64, 128, 96, 31), latent(16, 16, 8, 24, 33, 20, 65),
           latent(17, 20, 12, 28, 40, 36, 100), latent(3, 65, 66, 129, 130, 7, 32),
           latent(2, 128, 64, 128, 300, 200, 90), latent(40, 10, 4, 12, 20, 65, 70),
           latent(2, 33, 100, 40, 512, 64, 1000, 100.0, 0.02),
           latent(3, 128, 128, 70, 500, 64, 149)]


@pytest.mark.parametrize("k", range(len(LATENTS)))
def test_latent_attention_alone(k):
    check_alone(config([(LATENTS[k], None)]), seed=k)


@pytest.mark.parametrize("ff", [1, 40, 64, 200, 5000])
def test_dense_alone(ff):
    """A mixer that writes nothing: its post norm leaves 0."""
    cfg = config([(latent(), dense(ff))], width=72)
    w = weights(cfg)
    w["l0.mix.o"] *= 0
    check_alone(cfg, 90, cuts=([90], [1] * 90, [23, 2, 65]), w=w)


@pytest.mark.parametrize("E, top, shared, ff", [
    (5, 2, 72, 40), (1, 1, None, 64), (8, 1, 8, 200), (3, 3, 130, 16),
    (70, 4, None, 24), (130, 9, 40, 8)])
def test_experts_alone(E, top, shared, ff):
    """Every size class of the batch, by the worst row in fp32; bf16 over
    the rows whose choice is clear."""
    cfg = config([(latent(), moe(E, top, ff, shared))], width=72)
    w = weights(cfg)
    w["l0.mix.o"] *= 0
    t = tokens(cfg, 190)
    gap = []

    def choose(z, top, real=O.choose):
        s = np.sort(z)[::-1]
        gap.append(s[top - 1] - s[top] if top < len(s) else 9.0)
        return real(z, top)
    O.choose, keep = choose, O.choose
    try:
        want, _ = Oracle(cfg, w).run(t)
    finally:
        O.choose = keep
    m, clear = engine(cfg, w), np.array(gap) > 0.08
    assert clear.sum() > 20 and min(gap) > 1e-5
    cuts = [190], [1] * 190, [4, 6, 23, 60, 97]
    for c in cuts:
        assert worst(run(m, t, c), want) < EXACT, c
    for rows in (2, 5, 9, 19):                 # decode batches
        m = engine(cfg, w, max_batch=rows)
        seqs = [m.open_sequence() for _ in range(rows)]
        got = m.step([entry(s, t[k:k + 1]) for k, s in enumerate(seqs)])
        alone = [Oracle(cfg, w).run(t[k:k + 1])[0][0] for k in range(rows)]
        assert worst(got.cpu().numpy(), np.stack(alone)) < EXACT
    m = engine(cfg, w, "bf16")
    for c in cuts:
        assert rel(run(m, t, c)[clear], want[clear]) < ROUNDED, c


@pytest.mark.parametrize("kw", [dict(width=64, vocab=64), dict(width=130),
                                dict(eps=0.3), dict(vocab=1001), dict(emb=16.0),
                                dict(width=520), dict(taps=1), dict(taps=2),
                                dict(taps=7), dict(taps=12)])
def test_stack_constants(kw):
    cfg = config([(latent(), dense(50)), (latent(2), None),
                  (latent(4), moe()), (latent(), dense(50), 0)], **kw)
    w, t = weights(cfg), tokens(cfg, 41)
    want, _ = Oracle(cfg, w).run(t)
    m = engine(cfg, w)
    for c in ([41], [1] * 41, [2, 10, 2, 1, 26]):
        assert worst(run(m, t, c), want) < EXACT


def test_shared_tensors_keep_their_own_cache():
    cfg = config([(latent(), dense(50)), (latent(), dense(50), 0),
                  (latent(), dense(50), 1)])
    w, t = weights(cfg), tokens(cfg, 80)
    want, _ = Oracle(cfg, w).run(t)
    m = engine(cfg, w)
    assert len(m.caches) == 3 and len(m.layers) == 1
    assert len({c[0].data_ptr() for c in m.caches}) == 3
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


def test_bf16_whole_model():
    """All experts chosen, so that no close call decides."""
    cfg = config([(latent(), dense()), (latent(5, 12, 8, 16, 70, 52, 64),
                                        moe(3, 3)), (latent(), dense(), 0)])
    w, t = weights(cfg), tokens(cfg, 300)
    want, _ = Oracle(cfg, w).run(t)
    m = engine(cfg, w, "bf16")
    for sizes in ([300], [1], [2, 70, 1]):
        assert rel(run(m, t, cut(300, sizes)), want) < ROUNDED


def test_long_prompt_with_split_keys():
    """Later portions of a long prompt: key splits of runs and tokens, with
    windows that begin inside the cache and one that never does."""
    cfg = config([(latent(8, 24, 12, 40, 64, 36, 1100), None),
                  (latent(2, window=2000), None), (latent(6, window=300), None)])
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


@pytest.mark.parametrize("window", [2, 3, 31, 32, 33, 63, 64, 65, 100, 136])
@pytest.mark.parametrize("heads", [1, 4, 20])
def test_window_edges(window, heads):
    """The key that stands out is the last one seen, or the first one not;
    the asking token comes at every place of pages and tiles."""
    for end in (140, 143, 159, 160, 161, 191, 192):
        for back in (window - 1, window):
            cfg, w, t = needle(end - back, end + 1, window, heads)
            want = Oracle(cfg, w).run(t)[0][-1:]
            m = engine(cfg, w)
            for cuts in ([end + 1], [end, 1], [end - 1, 2], [end - 30, 31]):
                assert worst(run(m, t, cuts)[-1:], want) < EXACT, (end, cuts)


def test_window_passes_over_decoded_tokens():
    """The asking token at every distance while decoding: 20 of them see
    the key, the ones after do not."""
    cfg, w, t = needle(100, 200, 21, 3)
    o = Oracle(cfg, w)
    m = engine(cfg, w)
    seqs = [m.open_sequence() for _ in range(2)]
    m.step([entry(s, t[:95], []) for s in seqs])
    _, st = o.run(t[:95])
    seen = []
    for k in range(95, 150):
        ask = 1 if k == 100 else 2
        z, st2 = o.run([ask], st)
        got = m.step([entry(seqs[0], [ask])]).cpu().numpy()
        assert worst(got, z) < EXACT, k
        seen.append(z[0])
        # the second sequence goes on beside it, two tokens at a time
        if k % 2:
            m.step([entry(seqs[1], [2, 2], [])])
        st = st2
    seen = np.array(seen) - seen[-1]
    d = np.abs(seen).max(-1)
    assert d[6:26].min() > 100 * d[27:].max()


def test_far_key_while_decoding():
    """The asking token comes at every place after a long decode."""
    cfg, w, t = needle(5, 200, 500, 6)
    o = Oracle(cfg, w)
    m = engine(cfg, w)
    s = m.open_sequence()
    m.step([entry(s, t[:10], [])])
    _, st = o.run(t[:10])
    for k in range(10, 150):
        ask = 2 if k % 9 == 0 else int(t[k])
        z, st = o.run([ask], st)
        got = m.step([entry(s, [ask])]).cpu().numpy()
        assert worst(got, z) < EXACT, k


@pytest.mark.parametrize("sink", [-200.0, 0.0, 8.0, 200.0])
def test_sinks_at_their_extremes(sink):
    """A sink that never counts, one among the scores, one that takes all
    (and must not overflow); with few and with many keys."""
    cfg = config([(latent(5, window=70), None)])
    w, t = weights(cfg), tokens(cfg, 120)
    w["l0.mix.sink"][:] = sink
    w["l0.mix.sink"][2] = 1.0
    want, _ = Oracle(cfg, w).run(t)
    m = engine(cfg, w)
    for cuts in ([120], [1] * 120, [50, 2, 1, 67]):
        assert worst(run(m, t, cuts), want) < EXACT


@pytest.mark.parametrize("sub", ["canon1", "canon2"])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 6])
def test_convolution_window(taps, sub):
    """With a mixer that sees one token and the oldest tap as large as the
    rest, an input one place off or lost at a cut shows in the row that
    should see it last, and not in the next."""
    cfg = config([(latent(window=1), dense(40))], taps=taps)
    w, t = weights(cfg, 3), tokens(cfg, 80)
    for name in ("canon1", "canon2"):
        w["l0." + name] *= 0
    w["l0." + sub][:, 0] = 2.0
    o = Oracle(cfg, w)
    want, _ = o.run(t)
    p = 40
    other = t.copy()
    other[p] = (t[p] + 7) % cfg["vocab"]
    diff = np.abs(o.run(other)[0] - want).max(-1)
    assert diff[p + taps - 1] > 0.05 and diff[p + taps:].max() < 1e-6
    m = engine(cfg, w)
    for k in range(p, p + taps + 1):           # a cut at every place
        for cuts in ([k, 80 - k], [k] + [1] * (80 - k), [k, 2, 78 - k]):
            assert worst(run(m, t, cuts), want) < EXACT
            assert worst(run(m, other, cuts), o.run(other)[0]) < EXACT


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


def test_rewind_where_nothing_is_carried_along():
    cfg = config([(latent(), dense(40)), (latent(2), moe(4, 4))], taps=1)
    w, t = weights(cfg), tokens(cfg, 40)
    m = engine(cfg, w)
    m.prefill(t)
    m.rewind(25)
    want, _ = Oracle(cfg, w).run(np.concatenate([t[:25], t[:9]]))
    assert worst(m.forward_positions(t[:9], 25), want[25:]) < EXACT


def test_server_batches_requests(tmp_path):
    """The HTTP scheduler: concurrent greedy requests in one lockstep
    group give what each gives alone."""
    pytest.importorskip("fastapi")
    from concurrent.futures import ThreadPoolExecutor

    from fastapi.testclient import TestClient

    from llm_np_cp_amd.runtime.server import build_app

    cfg = config([(latent(), dense(60)), (latent(2), moe()),
                  (latent(), dense(60), 0)], vocab=280)
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
    cfg = config([(latent(), dense(60)), (latent(2), moe())], vocab=300)
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
    cfg = config([(latent(), dense()), (latent(5, 12, 8, 16, 70, 52, 64),
                                        moe(3, 3)), (latent(), dense(), 0)])
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
