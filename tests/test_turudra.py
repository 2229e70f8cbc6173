"""Turudra without a GPU: configuration, tensors, registry, cache
bookkeeping, and the oracle's own consistency."""

import json

import numpy as np
import pytest

from turudra_cases import (config, default, greedy, latent, mlstm, moe, rel,
                           save, tokens, weights)
from turudra_oracle import Oracle, layer_runs


def test_config_roundtrip_and_runs():
    from llm_np_cp_amd.core.config import ModelConfig
    from llm_np_cp_amd.core.layered import LayeredConfig

    d = default()
    c = ModelConfig.from_hf_dict(d)
    assert isinstance(c, LayeredConfig) and c.to_dict() == d
    assert c.runs == layer_runs(d)
    assert (c.model_type, c.vocab_size, c.hidden_size) == ("turudra", 157, 88)
    assert c.recurrent and c.is_moe and c.eos_token_id is None
    plain = ModelConfig.from_hf_dict(config([(latent(), None)]))
    assert not plain.recurrent and not plain.is_moe
    assert plain.runs == [(0, False)]


@pytest.mark.parametrize("change, text", [
    (lambda d: d.update(architecture="Other"), "architecture"),
    (lambda d: d["layers"][0].update(type="conv"), "unknown mixer"),
    (lambda d: d["layers"][0]["mlp"].update(kind="dense"), "feed-forward"),
    (lambda d: d["layers"][0]["mixer"].pop("kv_rank"), "kv_rank"),
    (lambda d: d["layers"][0]["mixer"].update(heads=0), "heads"),
    (lambda d: d["layers"][0]["mixer"]["rot"].update(dims=14), "rot.dims"),
    (lambda d: d["layers"][0]["mlp"]["router"].update(top=9), "top 9"),
    (lambda d: d.update(loop={"start": 2, "stop": 9, "times": 1}), "loop"),
    (lambda d: d.pop("norm"), "norm")])
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
    assert np.array_equal(lazy["l1.mix.i.b"], w["l1.mix.i.b"])
    for name in ("loop.in", "l0.mix.dkv.norm", "l1.mlp.e3.down",
                 "l0.mlp.shared.gate", "l2.mix.uk", "head"):
        assert name in w
    assert "l2.mlp.router" not in w and "l3.mlp.shared.gate" not in w
    bad = dict(w)
    bad.pop("l0.mix.uv")
    with pytest.raises(ValueError, match="l0.mix.uv"):
        validate_weights(cfg, bad)


def test_presets_and_registry():
    import llm_np_cp_amd as L
    from llm_np_cp_amd.core.config import has_preset, preset_names
    from llm_np_cp_amd.models import registry

    assert has_preset("tiny-turudra") and "tiny-turudra" in preset_names()
    cfg = L.preset_config("tiny-turudra")
    assert registry.engine_class(cfg).__name__ == "LayeredModel"
    assert registry.engine_class(L.preset_config("tiny-llama")).__name__ == \
        "GPUModel"
    with pytest.raises(ValueError, match="no CPU backend"):
        L.load_model("tiny-turudra", backend="numpy")


def test_engine_refuses_what_it_cannot_do():
    import llm_np_cp_amd as L
    from llm_np_cp_amd.models.layered import LayeredModel

    cfg = L.preset_config("tiny-turudra")
    with pytest.raises(ValueError, match="bf16 or fp32"):
        LayeredModel(cfg, {}, dtype="fp8")
    with pytest.raises(ValueError, match="kv_dtype"):
        LayeredModel(cfg, {}, kv_dtype="fp8")

    class Recurrent:
        no_rewind, config = True, cfg

    with pytest.raises(ValueError, match="recurrent"):
        L.generate_speculative("x", L.ByteTokenizer(), Recurrent(),
                               Recurrent())


def test_cache_manager_reuses_pages_and_slots():
    from llm_np_cp_amd.runtime.cache_manager import CacheFull, CacheManager

    c = CacheManager(pages=5, slots=2, page_size=64)
    a, b = c.open(), c.open()
    with pytest.raises(CacheFull):
        c.open()
    c.reserve(a, 65)
    c.reserve(b, 128)
    assert c.free_pages == 1 and not set(a.pages) & set(b.pages)
    assert list(c.table[a.slot, :2]) == a.pages
    v = c.version
    c.reserve(a, 128)                       # already has room
    assert c.version == v
    with pytest.raises(CacheFull):
        c.reserve(a, 64 * 4)
    assert c.free_pages == 1 and len(a.pages) == 2      # nothing changed
    freed, slot = set(a.pages), a.slot
    c.close(a)
    with pytest.raises(ValueError):
        c.close(a)
    with pytest.raises(ValueError):
        c.reserve(a, 1)
    n = c.open()
    assert n.slot == slot
    c.reserve(n, 3 * 64)
    assert freed <= set(n.pages) and c.free_pages == 0
    c.close_all()
    assert c.free_pages == 5 and c.free_slots == 2


def test_cache_manager_random_walk():
    from llm_np_cp_amd.runtime.cache_manager import CacheFull, CacheManager

    rng = np.random.default_rng(3)
    c, live = CacheManager(pages=12, slots=4, page_size=16), {}
    for _ in range(600):
        if live and rng.random() < 0.3:
            c.close(live.pop(rng.choice(list(live))))
        elif c.free_slots and rng.random() < 0.5:
            s = c.open()
            live[s.slot] = s
        elif live:
            s = live[rng.choice(list(live))]
            n = s.length + int(rng.integers(1, 40))
            try:
                c.reserve(s, n)
                s.length = n
            except (CacheFull, ValueError):
                assert c.missing(s, n) > 0
        held = [p for s in live.values() for p in s.pages]
        assert len(held) == len(set(held)) == 12 - c.free_pages
        for s in live.values():
            assert s.length <= 16 * len(s.pages)
            assert list(c.table[s.slot, :len(s.pages)]) == s.pages


def test_single_request_cannot_exceed_its_table_row():
    from llm_np_cp_amd.runtime.cache_manager import CacheManager

    c = CacheManager(pages=8, slots=2, page_size=64, max_seq=128)
    s = c.open()
    with pytest.raises(ValueError, match="exceed"):
        c.reserve(s, 129)


def test_oracle_portions_equal_whole():
    """The reference itself: any cut of the tokens gives the same logits."""
    d = default()
    o, t = Oracle(d, weights(d)), tokens(d, 37)
    whole, _ = o.run(t)
    for cuts in ([1] * 37, [2, 3, 30, 2], [36, 1]):
        st, out, at = None, [], 0
        for n in cuts:
            z, st = o.run(t[at:at + n], st)
            out.append(z)
            at += n
        assert rel(np.concatenate(out), whole) < 1e-12


@pytest.mark.parametrize("kind", ["mask", "gate", "rotation", "forget",
                                  "shared", "loop"])
def test_planted_mistakes_show(kind, monkeypatch):
    """Corrupting one mechanism of the oracle moves its logits far beyond
    the tolerances the GPU tests use, so those tests can notice."""
    import turudra_oracle as T

    d = default()
    w, t = weights(d), tokens(d, 40)
    want, _ = Oracle(d, w).run(t)
    w2, d2 = dict(w), json.loads(json.dumps(d))
    if kind == "mask":         # a token sees one step less
        real = T.latent_attention

        def late(w, p, m, h, eps, st):
            y, s = real(w, p, m, h, eps, st)
            return np.concatenate([y[:1], y[:-1]]), s
        monkeypatch.setitem(T.MIXERS, "latent_attention", late)
    elif kind == "gate":
        w2["l0.mix.g"] = w["l0.mix.g"] * 0
    elif kind == "rotation":
        for l in (0, 2):
            d2["layers"][l]["mixer"]["rot"]["base"] *= 3
    elif kind == "forget":
        w2["l1.mix.f.b"] = w["l1.mix.f.b"] + 1.5
    elif kind == "shared":
        d2["layers"][0]["mlp"]["shared"]["limit"] *= 2
    elif kind == "loop":
        w2["loop.in"] = w["loop.in"] * (np.arange(2 * 88) < 88)
    got, _ = Oracle(d2, w2).run(t)
    assert rel(got, want) > 3e-2


def test_greedy_oracle_is_deterministic():
    d = config([(mlstm(), moe())])
    w = weights(d)
    assert greedy(d, w, tokens(d, 5), 6)[0] == greedy(d, w, tokens(d, 5), 6)[0]


def test_trace_run_refuses_other_families(tmp_path):
    from llm_np_cp_amd.io.loader import write_synthetic_checkpoint
    from llm_np_cp_amd.runtime.trace import main

    write_synthetic_checkpoint(str(tmp_path), "tiny-llama")
    assert main(["--model", str(tmp_path), "--dtype", "bfloat16", "--out",
                 str(tmp_path), "--max-tokens", "64"]) == 2
