"""Model families: what a config's architecture name selects -- the model class, the processor, the weight table."""
import importlib


class Family:
    """`units`: the translation units (csrc/p3v_<unit>.hip) a program that runs only this family needs; None = all of them."""

    def __init__(self, name, model, processor, weight_specs, layered=False, units=None):
        self.name, self.model_ref, self.processor_ref, self.specs_ref = name, model, processor, weight_specs
        self.layered, self.units = layered, units

    @staticmethod
    def _get(ref):
        mod, attr = ref.split(":")
        return getattr(importlib.import_module("." + mod, __package__), attr)

    @property
    def model_cls(self):
        return self._get(self.model_ref)

    @property
    def processor_cls(self):
        return self._get(self.processor_ref)

    def weight_specs(self, cfg):
        return self._get(self.specs_ref)(cfg)


FAMILIES = [
    Family("Phi3V", "model:Phi3VModel", "processor:Phi3VProcessor", "weights:phi3_weight_specs"),
    Family("Phi3F", "model:Phi3VModel", "processor:Phi3FProcessor", "weights:phi3_weight_specs"),
    Family("Pelalix", "layered:LayeredModel", "processor:TextProcessor", "weights:layered_weight_specs", layered=True,
           units=("elementwise", "gemm", "gemm256", "gemm_skinny", "gemm_rows", "gemv", "layered", "attn_mix", "runtime")),
    Family("Pudisun", "layered:LayeredModel", "processor:TextProcessor", "weights:layered_weight_specs", layered=True,
           units=("elementwise", "gemm", "gemm256", "gemm_skinny", "gemm_rows", "gemv", "layered", "latent", "latent_prompt", "gla", "runtime")),
]


def family_of_name(arch):
    """`architectures[0]` / `architecture` of a config.json -> Family.  (Phi-3 names keep the reference's rule: Phi3V* is the vision
    model, any other Phi3* the text model.)"""
    for f in FAMILIES:
        if arch == f.name or (f.name == "Phi3V" and arch.startswith("Phi3V")):
            return f
    if arch.startswith("Phi3"):
        return FAMILIES[1]
    raise ValueError(f"unknown architecture {arch!r}; known: {', '.join(f.name for f in FAMILIES)}")


def family(cfg):
    return family_of_name(cfg.architectures[0])
