from .attention import paged_decode_attention, store_kvcache  # noqa: F401
from .fused import qk_norm_rope_store, rms_norm, silu_and_mul  # noqa: F401
from .latent import LatentAttention, latent_rows_attention, latent_tiles_attention  # noqa: F401
from .residual import embed_norm, residual_norm, xielu  # noqa: F401
