from .decoder import DecoderModel, LayerRun, LoopInputs, TokenEmbedding, OutputHead
from .qwen3 import build_qwen3
from .bizipel import build_bizipel
from .kamivik import build_kamivik
from .repolix import build_repolix
from .nilepel import build_nilepel
from .pizunex import build_pizunex
from .sunosun import build_sunosun

__all__ = ["DecoderModel", "LayerRun", "LoopInputs", "TokenEmbedding", "OutputHead", "build_qwen3", "build_bizipel", "build_kamivik", "build_repolix",
           "build_nilepel", "build_pizunex", "build_sunosun"]
