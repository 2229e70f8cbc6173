"""Model classes by configuration.

``engine_class(config)`` is the GPU engine that serves a config,
``oracle_class(config)`` the NumPy model of the CPU backend (None where a
design has no CPU backend).  A new design registers its ``model_type``
here; loading, generation, serving and the trace runner go through these.
"""

from __future__ import annotations


def _dense():
    from .engine import GPUModel
    return GPUModel


def _layered():
    from .layered import LayeredModel
    return LayeredModel


def _numpy():
    from .numpy_ref import NumpyModel
    return NumpyModel


# model_type -> (GPU engine, NumPy oracle, kernel libraries of its forward
# pass; None: the config names them)
MODELS = {t: (_dense, _numpy, ("llmops",))
          for t in ("llama", "gemma2", "qwen2", "mistral", "mixtral")}
MODELS.update({t: (_layered, None, None)
               for t in ("turudra", "garupel", "fidizen", "dogalorn")})


def _entry(config):
    if config.model_type not in MODELS:
        raise ValueError(f"no model class for {config.model_type!r}; have "
                         f"{sorted(MODELS)}")
    return MODELS[config.model_type]


def engine_class(config):
    return _entry(config)[0]()


def oracle_class(config):
    make = _entry(config)[1]
    return make() if make else None


def kernel_libraries(config):
    return _entry(config)[2] or config.kernel_libraries()
