from . import fopinex  # registers Fopinex
from . import getodra  # registers Getodra
from . import nosedra  # registers Nosedra
from . import qwen2_moe  # registers Qwen2MoeForCausalLM
from . import rudazen  # registers Rudazen
from . import sosepel  # registers Sosepel
from . import tuzapel  # registers Tuzapel
from .spec import LayerCall, ModelSpec

__all__ = ["LayerCall", "ModelSpec", "fopinex", "getodra", "nosedra", "qwen2_moe", "rudazen", "sosepel", "tuzapel"]
