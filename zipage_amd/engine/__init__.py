from .config import EngineConfig  # noqa: F401
from .kapolorn import Kapolorn, KapolornShape  # noqa: F401
from .llm import ZipageEngine  # noqa: F401
from .mefupel import Mefupel, MefupelShape  # noqa: F401
from .pages import PagePool  # noqa: F401
from .pedivik import Pedivik, PedivikLayer, PedivikShape  # noqa: F401
from .qwen3 import QWEN3_0_6B, QWEN3_8B, Qwen3, Qwen3Shape, StepContext  # noqa: F401
from .registry import ARCHITECTURES, build_model, read_shape  # noqa: F401
from .rutevik import Rutevik, RutevikShape  # noqa: F401
from .scheduler import Scheduler  # noqa: F401
from .sequence import Portion, SamplingParams, Sequence  # noqa: F401
