"""What the GPU tests of the layer-list designs share: an engine whose
caches start as NaN, so reading a position or a state that the sequence
has not written fails a comparison, and ways to feed it."""

import numpy as np

EXACT = 2e-4        # fp32 engine against float64, worst row
ROUNDED = 6e-2      # bf16 engine, all rows together


def engine(cfg, w, dtype="fp32", max_seq=320, max_batch=4, **kw):
    from llm_np_cp_amd.core.layered import LayeredConfig
    from llm_np_cp_amd.models.layered import LayeredModel

    m = LayeredModel(LayeredConfig.from_dict(cfg), w, dtype=dtype,
                     max_seq=max_seq, max_batch=max_batch, **kw)
    def spoil(c):
        if isinstance(c, tuple):
            for t in c:
                spoil(t)
        else:
            c.fill_(float("nan"))
    spoil(tuple(m.caches))
    return m


def entry(seq, toks, want=None):
    from llm_np_cp_amd.models.layered import StepEntry
    return StepEntry(seq, toks, range(len(toks)) if want is None else want)


def run(m, t, cuts=None):
    """Logits of every token of t fed in portions of the given sizes."""
    s, out, at = m.open_sequence(), [], 0
    for n in cuts or [len(t)]:
        out.append(m.step([entry(s, t[at:at + n])]).cpu().numpy())
        at += n
    assert at == len(t)
    m.close_sequence(s)
    return np.concatenate(out)


def cut(total, sizes):
    out, i = [], 0
    while sum(out) < total:
        out.append(min(sizes[i % len(sizes)], total - sum(out)))
        i += 1
    return out
