from .attention import paged_decode_attention, store_kvcache  # noqa: F401
from .fused import qk_norm_rope_store, rms_norm, silu_and_mul  # noqa: F401
from .grouped import GroupedAttention, grouped_rows_attention, rotary_store, store_form  # noqa: F401
from .latent import LatentAttention, rotate_heads, latent_rows_attention, latent_tiles_attention  # noqa: F401
from .moe import Experts, small_linear  # noqa: F401
from .recurrent import ChannelDelta, LinearAttention, MatrixMemory  # noqa: F401
from .residual import embed_norm, normed_powers, relu_square, residual_norm, softcap, xielu  # noqa: F401
from .rotary import Rotary  # noqa: F401
from .runs import attention_form, gather_rows, run_attention  # noqa: F401
