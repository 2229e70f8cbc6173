"""Dogalorn without a GPU: configuration, tensors, registry, distance
buckets, and the oracle's own consistency."""

import json

import numpy as np
import pytest

from dogalorn_cases import (attention, config, default, dense, greedy, memory,
                            needle, pair, rel, save, ssd, tokens, weights, worst)
from dogalorn_oracle import Oracle, bucket, owner


def test_config_roundtrip_and_runs():
    from llm_np_cp_amd.core.config import ModelConfig
    from llm_np_cp_amd.core.layered import LayeredConfig

    d = default()
    c = ModelConfig.from_hf_dict(d)
    assert isinstance(c, LayeredConfig) and c.to_dict() == d
    assert [i for i, _ in c.runs] == [owner(d, i) for i in range(8)]
    assert [i for i, _ in c.runs] == [0, 1, 2, 3, 0, 0, 1, 7]
    assert (c.model_type, c.vocab_size, c.hidden_size) == ("dogalorn", 157, 88)
    assert (c.streams, c.logit_scale, c.bigram.buckets) == (3, 0.6, 211)
    assert c.recurrent and not c.is_moe and c.eos_token_id is None
    one = ModelConfig.from_hf_dict(config([(ssd(), None)], streams=1))
    assert one.streams == 1 and one.recurrent


@pytest.mark.parametrize("change, text", [
    (lambda d: d["layers"][0].update(type="attention"), "unknown mixer"),
    (lambda d: d["layers"][0]["mlp"].update(kind="moe"), "feed-forward"),
    (lambda d: d["layers"][0]["mixer"].pop("right"), "right"),
    (lambda d: d["layers"][0]["mixer"]["right"].pop("width"), "width"),
    (lambda d: d["layers"][0]["mixer"]["left"].pop("scale"), "scale"),
    (lambda d: d["layers"][0]["mixer"]["left"].pop("mask"), "mask"),
    (lambda d: d["layers"][0]["mixer"]["left"]["mask"].update(size=0),
     "mask.size"),
    (lambda d: d["layers"][0]["mixer"]["left"].update(vdim=24), "vdim 24"),
    (lambda d: d["layers"][0]["mixer"]["left"].update(kv_heads=3), "kv_heads"),
    (lambda d: d["layers"][0]["mixer"]["left"].update(bias_max=0), "bias_max"),
    (lambda d: d["layers"][1]["mixer"].update(groups=4), "groups"),
    (lambda d: d["layers"][1]["mixer"].update(norm_groups=7), "norm_groups"),
    (lambda d: d["layers"][1]["mixer"].pop("conv"), "conv"),
    (lambda d: d.pop("streams"), "streams"),
    (lambda d: d.update(streams=0), "streams"),
    (lambda d: d.pop("logit_scale"), "logit_scale"),
    (lambda d: d["embedding"].pop("bigram"), "bigram"),
    (lambda d: d["embedding"]["bigram"].update(buckets=0), "buckets"),
    (lambda d: d.update(loop={"start": 0, "stop": 1, "times": 2}), "loop"),
    (lambda d: d["layers"][4].update(weights_of=4), "weights_of"),
    (lambda d: d["layers"][4].update(weights_of=2), "differs")])
def test_config_errors_name_the_key(change, text):
    from llm_np_cp_amd.core.layered import LayeredConfig

    d = json.loads(json.dumps(default()))
    change(d)
    with pytest.raises(ValueError, match=text):
        LayeredConfig.from_dict(d)


def test_weight_names_and_validation(tmp_path):
    from llm_np_cp_amd.io.loader import (LazyCheckpointWeights, load_config,
                                         validate_weights)

    d = default()
    w = weights(d)
    save(d, w, tmp_path / "m")
    cfg = load_config(str(tmp_path / "m"))
    lazy = LazyCheckpointWeights(str(tmp_path / "m"))
    validate_weights(cfg, lazy)
    assert np.array_equal(lazy["l0.mix.left.rel"], w["l0.mix.left.rel"])
    assert lazy["l0.norm1"].shape == w["final.norm"].shape == ()
    shapes = {"bigram": (212, 88), "l0.hc1.in": (3,), "l0.hc2.mix": (3, 3),
              "l0.mix.left.q.norm": (80,), "l0.mix.left.k.norm": (40,),
              "l0.mix.left.rel": (10, 4), "l0.mix.left.temp": (4,),
              "l0.mix.left.out": (88,), "l0.mix.right.z.b": (92,),
              "l0.mix.right.g": (92, 88), "l0.mlp.up.b": (112,),
              "l0.mlp.down.b": (88,), "l1.mix.in": (120 + 288 + 6, 88),
              "l1.mix.conv": (288, 4), "l1.mix.conv.b": (288,),
              "l1.mix.A_log": (6,), "l1.mix.D": (6,), "l1.mix.norm": (120,)}
    assert {k: w[k].shape for k in shapes} == shapes
    for name in ("l0.mix.left.v", "l0.mix.left.g", "l2.norm2", "l2.hc2.in",
                 "l0.mix.right.g.b", "l4.norm1", "l4.hc1.in", "l5.mix.left.q",
                 "l6.mix.in", "l7.mlp.up"):
        assert name not in w
    # the checkpoint decides the number of buckets, nothing else
    validate_weights(cfg, {**w, "l2.mix.left.rel": np.zeros((24, 3))})
    for bad in ({"l2.mix.left.rel": np.zeros((24, 4))},
                {"l0.mix.left.temp": np.zeros(5)}):
        with pytest.raises(ValueError, match=next(iter(bad))):
            validate_weights(cfg, {**w, **bad})
    bad = dict(w)
    bad.pop("l1.hc2.mix")
    with pytest.raises(ValueError, match="l1.hc2.mix"):
        validate_weights(cfg, bad)


def test_random_weights_scatter_around_something_useful():
    import llm_np_cp_amd as L
    from llm_np_cp_amd.io.loader import LazyRandomWeights, random_weights

    cfg = L.preset_config("tiny-dogalorn")
    for w in (random_weights(cfg), LazyRandomWeights(cfg)):
        assert abs(w["l0.norm1"] - 1) < 0.2 and w["l0.norm1"].shape == ()
        assert np.abs(w["l0.hc1.mix"] - np.eye(3)).max() < 0.2
        assert np.abs(w["l0.hc1.in"] - 1 / 3).max() < 0.2
        assert np.abs(w["l0.mix.left.out"] - 1).max() < 0.2
        assert np.abs(w["l0.mix.left.q"]).max() < 0.2
        assert all(w[k].dtype == np.float32 for k in w.keys())


def test_presets_registry_and_libraries():
    import llm_np_cp_amd as L
    from csrc.build import LIBS
    from llm_np_cp_amd.core.config import preset_names
    from llm_np_cp_amd.models import registry

    for name in ("tiny-dogalorn", "dogalorn-2k", "dogalorn-4k"):
        assert name in preset_names()
        cfg = L.preset_config(name)
        assert set(registry.kernel_libraries(cfg)) <= set(LIBS)
        assert L.ModelConfig.from_hf_dict(cfg.to_dict()).to_dict() == \
            cfg.to_dict()
    assert registry.engine_class(cfg).__name__ == "LayeredModel"
    with pytest.raises(ValueError, match="no CPU backend"):
        L.load_model("tiny-dogalorn", backend="numpy")
    libs = lambda layers: registry.kernel_libraries(
        L.ModelConfig.from_hf_dict(config(layers)))
    assert libs([(pair(), dense())]) == ("gqa", "linear", "mingru")
    assert libs([(ssd(), None)]) == ("linear", "ssd")


@pytest.mark.parametrize("rows, far", [
    (2, 1.5), (2, 9), (4, 3), (6, 17), (8, 100), (10, 30), (16, 128),
    (32, 128), (32, 36), (64, 1000), (20, 11)])
def test_distance_buckets(rows, far):
    """The table by distance against the plain buckets, and its end: the
    last entry holds for every distance beyond it."""
    from llm_np_cp_amd.models.mixers import distance_bias

    table = np.random.default_rng(rows).standard_normal((rows, 3))
    want = table[[bucket(n, rows, far) for n in range(1500)]].T
    got = distance_bias(table, far, 1500)
    assert got.shape[0] == 3 and got.shape[1] <= far + 2
    idx = np.minimum(np.arange(1500), got.shape[1] - 1)
    assert np.array_equal(got[:, idx], want)
    assert np.array_equal(distance_bias(table, far, 7), want[:, :7][
        :, :distance_bias(table, far, 7).shape[1]])
    for bad in (table[:1], table[:0], np.zeros((3, 2))):
        with pytest.raises(ValueError, match="buckets"):
            distance_bias(bad, far, 10)
    with pytest.raises(ValueError, match="buckets"):
        distance_bias(table, rows / 2, 10)


def test_oracle_portions_equal_whole():
    """The reference itself: any cut of the tokens gives the same logits."""
    for streams in (1, 2, 4):
        d = default(streams=streams)
        o, t = Oracle(d, weights(d)), tokens(d, 70)
        whole, _ = o.run(t)
        for cuts in ([1] * 70, [2, 3, 63, 2], [69, 1]):
            st, out, at = None, [], 0
            for n in cuts:
                z, st = o.run(t[at:at + n], st)
                out.append(z)
                at += n
            assert rel(np.concatenate(out), whole) < 1e-12


@pytest.mark.parametrize("kind", [
    "pair row", "pair order", "first row", "previous token", "mix direction",
    "read", "feed", "streams apart", "norm gain", "q norm per head",
    "values are normed keys", "no temperature", "scaled bias", "bias bucket",
    "bias sign", "sliding window", "chunk size", "no sink", "half sum",
    "half norm", "gru gate", "candidate", "gru output gate", "conv order",
    "conv bias", "no silu", "dt clamp", "dt bias", "decay", "input step",
    "groups", "skip", "gate after norm", "norm parts", "gelu", "up bias",
    "down bias", "own tensors", "logit scale"])
def test_planted_mistakes_show(kind, monkeypatch):
    """Corrupting one mechanism of the oracle moves its logits far beyond
    the tolerances the GPU tests use, so those tests can notice."""
    import dogalorn_oracle as O

    d = default()
    w, t = weights(d), tokens(d, 80)
    want, _ = Oracle(d, w).run(t)
    w2, d2 = dict(w), json.loads(json.dumps(d))
    patch = lambda name, fn: monkeypatch.setattr(O, name, fn)
    mixer = lambda i: d2["layers"][i]["mixer"]
    zero = lambda name: w2.update({name: w[name] * 0})
    if kind == "pair row":
        d2["embedding"]["bigram"]["mul_cur"] += 1
    elif kind == "pair order":
        b = d2["embedding"]["bigram"]
        b["mul_cur"], b["mul_prev"] = b["mul_prev"], b["mul_cur"]
    elif kind == "first row":
        real = O.embed
        patch("embed", lambda w, s, t, prev: real(
            w, s, t, 0 if prev is None else prev))
    elif kind == "previous token":       # two places back instead of one
        patch("embed", lambda w, s, t, prev: w["embed"][t] + w["bigram"][
            (np.roll(t, 2) * s["mul_prev"] + t * s["mul_cur"])
            % s["buckets"]])
    elif kind == "mix direction":
        w2.update({k: v.T for k, v in w.items() if k.endswith("mix")})
    elif kind == "read":
        w2["l0.hc1.in"] = w["l0.hc1.in"][::-1]
    elif kind == "feed":
        w2["l0.hc1.out"] = w["l0.hc1.out"][::-1]
    elif kind == "streams apart":        # the mix one stream after another
        def spread(xs, mix, out, y):
            xs = list(xs)
            for k in range(len(xs)):
                xs[k] = sum(mix[s, k] * xs[s] for s in range(len(xs))) + \
                    out[k] * y
            return xs
        patch("spread", spread)
    elif kind == "norm gain":
        w2["l0.norm1"] = w["l0.norm1"] * 0 + 1
    elif kind == "q norm per head":
        real = O.rms

        def rms(x, eps):
            if x.shape[-1] != 80:
                return real(x, eps)
            return real(x.reshape(-1, 4, 20), eps).reshape(x.shape)
        patch("rms", rms)
    elif kind == "values are normed keys":
        real = O.sink_softmax

        def att(w, p, m, h, eps, past):
            k = h @ w[p + "k"].T
            r = O.rms(k, eps) * w[p + "k.norm"]
            T, G, dim = len(h), m["kv_heads"], m["dim"]
            y, (kk, vv) = real_att(w, p, m, h, eps, past)
            q = (O.rms(h @ w[p + "q"].T, eps) * w[p + "q.norm"]).reshape(
                T, m["heads"], dim)
            out, kn = np.zeros_like(q), r.reshape(T, G, dim)
            for i in range(T):
                js = [j for j in range(i + 1)
                      if O.visible(i, j, m["mask"]["size"])]
                b = w[p + "rel"][[O.bucket(i - j, 10, m["bias_max"])
                                  for j in js]]
                for a in range(m["heads"]):
                    g = a // (m["heads"] // G)
                    s = kn[js, g] @ q[i, a] * m["scale"] * w[p + "temp"][a]
                    out[i, a] = real(s + b[:, a]) @ kn[js, g]
            return out.reshape(T, -1) @ w[p + "o"].T, (kk, vv)
        real_att = O.attention
        patch("attention", att)
    elif kind == "no temperature":
        w2["l0.mix.left.temp"] = w["l0.mix.left.temp"] * 0 + 1
    elif kind == "scaled bias":
        w2["l0.mix.left.rel"] = w["l0.mix.left.rel"] * mixer(0)["left"]["scale"]
    elif kind == "bias bucket":
        real = O.bucket
        patch("bucket", lambda n, rows, far: real(n + 1, rows, far))
    elif kind == "bias sign":
        w2["l0.mix.left.rel"] = -w["l0.mix.left.rel"]
    elif kind == "sliding window":
        patch("visible", lambda i, j, size: j <= i and i - j < size)
    elif kind == "chunk size":
        for l in d2["layers"]:
            if l["type"] == "parallel":
                l["mixer"]["left"]["mask"]["size"] += 1
    elif kind == "no sink":
        patch("sink_softmax", lambda s: np.exp(s) / np.exp(s).sum())
    elif kind == "half sum":
        real = O.halves
        patch("halves", lambda *a: 2 * real(*a))
    elif kind == "half norm":
        w2["l0.mix.right.out"] = w["l0.mix.right.out"] * 0 + 1
    elif kind == "gru gate":
        w2["l0.mix.right.z.b"] = w["l0.mix.right.z.b"] + 0.5
    elif kind == "candidate":
        patch("candidate", lambda u: u)
    elif kind == "gru output gate":
        w2["l0.mix.right.g"] = w["l0.mix.right.g"] * 0.5
    elif kind == "conv order":
        w2["l1.mix.conv"] = w["l1.mix.conv"][:, ::-1]
    elif kind == "conv bias":
        zero("l1.mix.conv.b")
    elif kind == "no silu":
        real = O.short_conv
        patch("short_conv", lambda *a: (lambda y, st: (y * 2, st))(*real(*a)))
    elif kind == "dt clamp":
        real = O.softplus
        patch("softplus", lambda z: np.maximum(real(z), 0.1))
    elif kind == "dt bias":
        zero("l1.mix.dt_bias")
    elif kind == "decay":
        w2["l1.mix.A_log"] = w["l1.mix.A_log"] + 0.5
    elif kind == "input step":
        real = O.softplus
        patch("softplus", lambda z: real(z) * 1.1)
    elif kind == "groups":
        n, C = 28 * 3, w["l1.mix.conv"]
        m = w["l1.mix.in"].copy()
        lo = 240
        m[lo:lo + n] = np.roll(m[lo:lo + n].reshape(3, 28, -1), 1,
                               0).reshape(n, -1)
        w2["l1.mix.in"] = m
    elif kind == "skip":
        zero("l1.mix.D")
    elif kind == "gate after norm":
        real = O.group_norm
        patch("group_norm", lambda y, g, n, eps: real(y, g, n, eps) * 0.8)
    elif kind == "norm parts":
        mixer(1)["norm_groups"] = 1
    elif kind == "gelu":
        patch("gelu", lambda z: z * O.sigmoid(1.702 * z))
    elif kind == "up bias":
        zero("l0.mlp.up.b")
    elif kind == "down bias":
        zero("l0.mlp.down.b")
    elif kind == "own tensors":          # layer 4 with layer 2's norm
        w2["l0.norm1"] = w["l2.norm1"]
    elif kind == "logit scale":
        d2["logit_scale"] = 1.0
    got, _ = Oracle(d2, w2).run(t)
    assert rel(got, want) > (2e-3 if kind == "gelu" else 1e-2)


@pytest.mark.parametrize("chunk", [40, 64])
def test_needle_shows_inside_and_only_inside_the_chunk(chunk):
    edge = 2 * chunk
    for at, seen in ((edge, True), (edge - 1, False)):
        cfg, w, t = needle(at, edge + chunk, chunk)
        want = Oracle(cfg, w).run(t)[0][-1:]
        gone = t.copy()
        gone[at] = 3
        off = worst(Oracle(cfg, w).run(gone)[0][-1:], want)
        assert off > 0.1 if seen else off < 1e-9


@pytest.mark.parametrize("kind", ["mingru", "ssd"])
def test_states_reach_back(kind):
    cfg, w, t = memory(kind, 200)
    other = t.copy()
    other[0] = 6
    o = Oracle(cfg, w)
    assert worst(o.run(other)[0][-1:], o.run(t)[0][-1:]) > 0.05


def test_greedy_oracle_is_deterministic():
    d = config([(pair(), dense(24)), (ssd(), dense())])
    w = weights(d)
    assert greedy(d, w, tokens(d, 5), 6)[0] == greedy(d, w, tokens(d, 5), 6)[0]
    assert attention()["vdim"] == attention()["dim"]
