"""Fidizen without a GPU: configuration, tensors, registry, and the
oracle's own consistency."""

import json

import numpy as np
import pytest

from fidizen_cases import (config, default, dense, greedy, latent, moe,
                           needle, rel, save, tokens, weights, worst)
from fidizen_oracle import Oracle, owner


def test_config_roundtrip_and_runs():
    from llm_np_cp_amd.core.config import ModelConfig
    from llm_np_cp_amd.core.layered import LayeredConfig

    d = default()
    c = ModelConfig.from_hf_dict(d)
    assert isinstance(c, LayeredConfig) and c.to_dict() == d
    assert [i for i, _ in c.runs] == [owner(d, i) for i in range(7)]
    assert [i for i, _ in c.runs] == [0, 1, 2, 0, 0, 1, 6]
    assert not any(add for _, add in c.runs)
    assert (c.model_type, c.vocab_size, c.hidden_size) == ("fidizen", 157, 88)
    assert c.num_hidden_layers == 7 and c.conv_taps == 3
    assert c.recurrent and c.is_moe and c.eos_token_id is None
    # one tap only weighs the current input: nothing is carried along
    one = ModelConfig.from_hf_dict(config([(latent(), dense())], taps=1))
    assert not one.recurrent and not one.is_moe
    # a layer may use the tensors of a later one
    later = ModelConfig.from_hf_dict(
        config([(latent(), None, 1), (latent(), None)]))
    assert [i for i, _ in later.runs] == [1, 1]


@pytest.mark.parametrize("change, text", [
    (lambda d: d["layers"][0].update(type="attention"), "unknown mixer"),
    (lambda d: d["layers"][0]["mlp"].update(kind="glu"), "feed-forward"),
    (lambda d: d["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda d: d["layers"][0]["mixer"].pop("q_rank"), "q_rank"),
    (lambda d: d["layers"][0]["mixer"].pop("mask"), "mask"),
    (lambda d: d["layers"][0]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda d: d["layers"][0]["mixer"]["rot"].update(dims=14), "rot.dims"),
    (lambda d: d["layers"][1]["mlp"]["router"].update(top=9), "top 9"),
    (lambda d: d["layers"][1]["mlp"]["expert"].pop("ff"), "ff"),
    (lambda d: d.pop("canon"), "canon"),
    (lambda d: d["canon"].update(taps=0), "taps"),
    (lambda d: d.update(loop={"start": 0, "stop": 1, "times": 2}), "loop"),
    (lambda d: d["layers"][3].update(weights_of=3), "weights_of"),
    (lambda d: d["layers"][0].update(weights_of=3), "weights_of"),
    (lambda d: d["layers"][3].update(weights_of=7), "weights_of"),
    (lambda d: d["layers"][3].update(weights_of=1), "differs")])
def test_config_errors_name_the_key(change, text):
    from llm_np_cp_amd.core.layered import LayeredConfig

    d = json.loads(json.dumps(default()))
    change(d)
    with pytest.raises(ValueError, match=text):
        LayeredConfig.from_dict(d)


def test_only_this_design_shares_tensors():
    import garupel_cases
    from llm_np_cp_amd.core.layered import LayeredConfig

    d = garupel_cases.default()
    d["layers"][3]["weights_of"] = 1
    with pytest.raises(ValueError, match="share"):
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
    assert np.array_equal(lazy["l1.mix.uq"], w["l1.mix.uq"])
    for name in ("l0.norm1", "l0.norm2", "l0.canon1", "l0.canon2", "l2.norm1",
                 "l0.mix.dq", "l0.mix.dq.norm", "l0.mix.sink", "l0.mlp.act",
                 "l1.mlp.router", "l1.mlp.shared.up", "l6.mlp.e5.down"):
        assert name in w
    for name in ("l0.norm1b", "l2.norm2", "l2.canon2", "l2.mlp.up",
                 "l0.mix.q", "l3.norm1", "l3.canon1", "l5.mlp.router",
                 "l6.mlp.shared.up"):
        assert name not in w
    assert w["l0.mix.g"].shape == (3 * 28, 88)
    bad = dict(w)
    bad.pop("l1.mix.sink")
    with pytest.raises(ValueError, match="l1.mix.sink"):
        validate_weights(cfg, bad)


def test_presets_registry_and_libraries():
    import llm_np_cp_amd as L
    from csrc.build import LIBS
    from llm_np_cp_amd.core.config import preset_names
    from llm_np_cp_amd.models import registry

    for name in ("tiny-fidizen", "fidizen-2k", "fidizen-4k"):
        assert name in preset_names()
        cfg = L.preset_config(name)
        assert set(registry.kernel_libraries(cfg)) <= set(LIBS)
    assert registry.engine_class(cfg).__name__ == "LayeredModel"
    with pytest.raises(ValueError, match="no CPU backend"):
        L.load_model("tiny-fidizen", backend="numpy")
    libs = lambda layers: registry.kernel_libraries(
        L.ModelConfig.from_hf_dict(config(layers)))
    assert libs([(latent(), dense())]) == ("latent", "linear")
    assert libs([(latent(), moe())]) == ("latent", "linear", "moe")


def test_oracle_portions_equal_whole():
    """The reference itself: any cut of the tokens gives the same logits."""
    for taps in (1, 3, 5):
        d = default(taps=taps)
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
    "window wide", "window narrow", "no sink", "scaled sink", "rotation pairs",
    "rotation base", "query norm", "latent norm", "gate per head", "gate",
    "conv order", "conv without input", "post norm", "pre norm",
    "cubes", "offset", "moments of z", "scores", "weights on outputs",
    "renormalised", "shared expert", "own tensors", "embedding"])
def test_planted_mistakes_show(kind, monkeypatch):
    """Corrupting one mechanism of the oracle moves its logits far beyond
    the tolerances the GPU tests use, so those tests can notice."""
    import fidizen_oracle as O

    d = default()
    w, t = weights(d), tokens(d, 80)
    want, _ = Oracle(d, w).run(t)
    w2, d2 = dict(w), json.loads(json.dumps(d))
    patch = lambda name, fn: monkeypatch.setattr(O, name, fn)
    if kind.startswith("window"):
        real, off = O.visible, 1 if kind == "window wide" else -1
        patch("visible", lambda p, n, win: real(p, n, win + off))
    elif kind == "no sink":
        real = O.sink_softmax
        patch("sink_softmax", lambda s, k: real(s, -np.inf))
    elif kind == "scaled sink":
        for l in d2["layers"]:
            w2.update({k: v * l["mixer"]["scale"] for k, v in w.items()
                       if k.endswith("sink")})
    elif kind == "rotation pairs":
        def halves(x, pos, base, dims):
            h = dims // 2
            a = pos[:, None] * base ** (-2.0 * np.arange(h) / dims)
            a = a.reshape((len(pos),) + (1,) * (x.ndim - 2) + (h,))
            u, v = x[..., :h], x[..., h:]
            return np.concatenate([u * np.cos(a) - v * np.sin(a),
                                   v * np.cos(a) + u * np.sin(a)], -1)
        patch("rotate", halves)
    elif kind == "rotation base":
        d2["layers"][0]["mixer"]["rot"]["base"] = 4e3
    elif kind == "query norm":
        w2["l0.mix.dq.norm"] = w["l0.mix.dq.norm"] * 0 + 1
    elif kind == "latent norm":
        w2["l0.mix.dkv.norm"] = w["l0.mix.dkv.norm"] * 0 + 1
    elif kind == "gate per head":
        w2["l0.mix.g"] = np.repeat(w["l0.mix.g"][::28], 28, axis=0)
    elif kind == "gate":
        w2["l0.mix.g"] = w["l0.mix.g"] * 0
    elif kind == "conv order":
        w2["l0.canon1"] = w["l0.canon1"][:, ::-1]
    elif kind == "conv without input":
        real = O.short_conv
        patch("short_conv", lambda h, k, b: (
            lambda y, s: (y - h, s))(*real(h, k, b)))
    elif kind == "post norm":
        w2["l0.norm2"] = w["l0.norm2"] * 0 + 1
    elif kind == "pre norm":
        real = O.short_conv
        patch("short_conv", lambda h, k, b: real(O.rms(h, 1e-5), k, b))
    elif kind == "cubes":
        w2["l0.mlp.act"] = w["l0.mlp.act"] * [1, 1, 0, 1]
    elif kind == "offset":
        w2["l0.mlp.act"] = w["l0.mlp.act"] * [1, 1, 1, 0]
    elif kind == "moments of z":
        def poly(z, c, eps):
            n = O.rms(z, eps)
            return c[0] * n + c[1] * n ** 2 + c[2] * n ** 3 + c[3]
        patch("polynorm", poly)
    elif kind == "scores":
        patch("choose", lambda z, top: (
            lambda i: (i, np.exp(z[i]) / np.exp(z[i]).sum()))(
                np.argsort(-z)[:top]))
    elif kind == "weights on outputs":
        def outside(w, p, m, h, eps):
            z, y = h @ w[p + "router"].T, np.zeros_like(h)
            for t in range(len(h)):
                for e, s in zip(*O.choose(z[t], m["router"]["top"])):
                    y[t] += s * O.expert(w, f"{p}e{e}.", h[t])
                if m.get("shared"):
                    y[t] += O.expert(w, p + "shared.", h[t])
            return y
        monkeypatch.setitem(O.FEED_FORWARDS, "moe", outside)
    elif kind == "renormalised":
        real = O.choose
        patch("choose", lambda z, top: (lambda i, s: (i, s / s.sum()))(
            *real(z, top)))
    elif kind == "shared expert":
        w2["l1.mlp.shared.down"] = w["l1.mlp.shared.down"] * 0
    elif kind == "own tensors":          # layer 3 runs with layer 2's norm
        w2["l0.norm1"] = w["l2.norm1"]
    elif kind == "embedding":
        d2["embedding"]["scale"] = 1.0
    got, _ = Oracle(d2, w2).run(t)
    assert rel(got, want) > 1e-2


@pytest.mark.parametrize("window", [40, 64])
def test_needle_shows_inside_and_only_inside_the_window(window):
    for back, seen in ((window - 1, True), (window, False)):
        cfg, w, t = needle(100 - back, 101, window)
        want = Oracle(cfg, w).run(t)[0][-1:]
        gone = t.copy()
        gone[100 - back] = 3
        off = worst(Oracle(cfg, w).run(gone)[0][-1:], want)
        assert off > 0.1 if seen else off < 1e-9


def test_greedy_oracle_is_deterministic():
    d = config([(latent(), dense(24)), (latent(), moe())])
    w = weights(d)
    assert greedy(d, w, tokens(d, 5), 6)[0] == greedy(d, w, tokens(d, 5), 6)[0]
