"""Which class serves a model folder.

A folder with a config.json names its design under "architecture"; the class registered for it reads the configuration
and the weights.  A folder in the reference's parameter format (no config.json, one file per projection and layer) is
Llama-3.2-1B in W8A8, or W4A4 on request."""
import importlib
import json
import os

from ._lib import ensure

# design -> module that registers it on import, the part of the library it needs
_MODULES = {"Lopazen": ("lopazen", "hybrid"), "Nifunex": ("nifunex", "hybrid")}
_CLASSES = {}


class UnknownModel(ValueError):
    pass


def register(name):
    def add(cls):
        _CLASSES[name] = cls
        return cls
    return add


def architectures():
    return sorted(_MODULES)


def model_class(name):
    if name not in _MODULES:
        raise UnknownModel("no model is registered for architecture %r (known: %s)" % (name, ", ".join(architectures())))
    module, component = _MODULES[name]
    ensure(component)
    importlib.import_module("." + module, __package__)
    return _CLASSES[name]


def load_model(path, dtype=None, max_pos=4096, slots=1, w4a4=False):
    """Model object of the folder `path`, ready to step and generate."""
    cfg_path = os.path.join(path, "config.json")
    if os.path.exists(cfg_path):
        with open(cfg_path) as f:
            cfg = json.load(f)
        cls = model_class(cfg.get("architecture"))
        return cls.from_dir(path, cfg, dtype=dtype or "bfloat16", max_pos=max_pos, slots=slots)
    if os.path.exists(os.path.join(path, "q_proj_L00.bin")):
        from . import llama, loader
        if dtype not in (None, "int8"):
            raise UnknownModel("the reference's parameter format is served in W8A8 or W4A4, not in %s" % dtype)
        cfg = llama.make_config(max_pos=max_pos)
        return llama.Llama(cfg, loader.load_reference_parameters(path, cfg, w4a4=w4a4))
    raise UnknownModel("%s holds neither a config.json nor parameters in the reference's format" % path)
