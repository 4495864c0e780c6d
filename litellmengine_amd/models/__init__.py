from . import qwen3  # noqa: F401  (registers Qwen3ForCausalLM)
from . import visadra  # noqa: F401  (registers Visadra)
from . import kezasun  # noqa: F401  (registers Kezasun)
from . import malilorn  # noqa: F401  (registers Malilorn)
from . import birelix  # noqa: F401  (registers Birelix)
from . import telulorn  # noqa: F401  (registers Telulorn)
from . import rorevik  # noqa: F401  (registers Rorevik)
from .build import expected_tensors, load_model, make_context, parse_dtype, random_model
from .decoder import DecoderLM, Inject, PlanEntry, looped_plan

__all__ = ["DecoderLM", "Inject", "PlanEntry", "expected_tensors", "load_model", "looped_plan", "make_context", "parse_dtype",
           "random_model"]
