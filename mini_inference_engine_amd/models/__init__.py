from . import llama  # noqa: F401  (registers LlamaForCausalLM)
from . import zifelorn  # noqa: F401  (registers Zifelorn)
from . import vezodra  # noqa: F401  (registers Vezodra)
from . import mutusun  # noqa: F401  (registers Mutusun)
from . import labirax  # noqa: F401  (registers Labirax)
from . import pokulorn  # noqa: F401  (registers Pokulorn)
from . import bulitar  # noqa: F401  (registers Bulitar)
from .decoder import Decoder
from .llama import build_llama
from .zifelorn import build_zifelorn
from .vezodra import build_vezodra
from .mutusun import build_mutusun
from .labirax import build_labirax
from .pokulorn import build_pokulorn
from .bulitar import build_bulitar
