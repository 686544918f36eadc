"""Decoder models and what they share. ``decoder``: the dense GQA + SwiGLU decoder the quantized
Linear layers sit in (the unchanged caller of the GEMM path; same modules, parameter names and math
as the reference's ``astrai/model``). ``lugitar`` and ``sarulix``: layers of different sequence mixers, built
from ``mixers``. ``registry`` picks the classes by config.json, ``cache`` is what a model keeps of its tokens."""

from astrai_amd.model.cache import MixerCache, RequestCaches, StepCache
from astrai_amd.model.decoder import (
    AutoRegressiveLM,
    AutoRegressiveLMConfig,
    DenseKVCache,
    fuse_int8_weights,
    greedy_generate,
    unfuse_int8_weights,
)
from astrai_amd.model.lugitar import LugitarConfig, LugitarLM
from astrai_amd.model.sarulix import SarulixConfig, SarulixLM
from astrai_amd.model.registry import architecture_of, architectures, register_architecture

from astrai_amd.model.checkpoint import (load_checkpoint, load_fp8_scaling, load_int8_checkpoint, save_fp8_scaling,
                                         save_int8_checkpoint)

__all__ = ["load_checkpoint", "load_fp8_scaling", "save_fp8_scaling", "load_int8_checkpoint", "save_int8_checkpoint",
           "AutoRegressiveLM", "AutoRegressiveLMConfig", "DenseKVCache", "greedy_generate", "fuse_int8_weights",
           "unfuse_int8_weights", "LugitarConfig", "LugitarLM", "SarulixConfig", "SarulixLM", "StepCache", "MixerCache", "RequestCaches",
           "architecture_of", "architectures", "register_architecture"]
