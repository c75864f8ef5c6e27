"""Model architectures the serving engine runs: configuration class and serving
class per architecture, chosen by ``config.json`` (``"architecture"``) or by the
type of a configuration object."""
from __future__ import annotations

import importlib
import json
from dataclasses import dataclass
from pathlib import Path


@dataclass(frozen=True)
class Architecture:
    name: str
    config: str   # "module:class"
    serving: str  # "module:class"

    @staticmethod
    def _get(ref: str):
        mod, _, cls = ref.partition(":")
        return getattr(importlib.import_module(mod), cls)

    def config_class(self):
        return self._get(self.config)

    def serving_class(self):
        return self._get(self.serving)


ARCHITECTURES = {a.name: a for a in (
    Architecture("Llama", "kgs.models.llama:LlamaConfig", "kgs.serve.model:ServingModel"),
    Architecture("Ruruzen", "kgs.models.ruruzen:RuruzenConfig", "kgs.serve.hybrid:HybridModel"),
    Architecture("Nufusun", "kgs.models.nufusun:NufusunConfig", "kgs.serve.nufusun:NufusunModel"),
    Architecture("Nokipel", "kgs.models.nokipel:NokipelConfig", "kgs.serve.nokipel:NokipelModel"),
    Architecture("Vumalix", "kgs.models.vumalix:VumalixConfig", "kgs.serve.vumalix:VumalixModel"),
)}


def of_config(cfg) -> Architecture:
    for a in ARCHITECTURES.values():
        if type(cfg).__module__ == a.config.partition(":")[0] and isinstance(cfg, a.config_class()):
            return a
    raise ValueError(f"no architecture is registered for {type(cfg).__name__}")


def load_config(folder):
    """The configuration of a model folder (``config.json`` beside ``model.safetensors``)."""
    d = json.loads((Path(folder) / "config.json").read_text())
    a = ARCHITECTURES.get(d.get("architecture"))
    if a is None or not hasattr(a.config_class(), "from_folder"):
        raise ValueError(f"{folder}: architecture {d.get('architecture')!r} has no checkpoint loader; "
                         f"known: {sorted(n for n, x in ARCHITECTURES.items() if hasattr(x.config_class(), 'from_folder'))}")
    return a.config_class().from_folder(folder)


def to_spec(cfg) -> dict:
    """A picklable description of ``cfg`` for a worker process."""
    import dataclasses

    return {"architecture": of_config(cfg).name,
            "spec": cfg.spec() if hasattr(cfg, "spec") else dataclasses.asdict(cfg)}


def from_spec(d: dict):
    """Inverse of :func:`to_spec`; plain fields are a Llama configuration's."""
    if "architecture" not in d:
        d = {"architecture": "Llama", "spec": d}
    cls = ARCHITECTURES[d["architecture"]].config_class()
    return cls.from_spec(d["spec"]) if hasattr(cls, "from_spec") else cls(**d["spec"])
