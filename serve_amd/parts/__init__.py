"""Parts of a layer.  Importing the package registers the standard kinds."""
from .base import (CacheTensor, LayerCache, ParamRequest, Part, PositionPart, Rotary, Runtime,  # noqa: F401
                   StateRequest, TokenCacheRequest, kv_cache_request)
from . import standard  # noqa: F401
from . import postnorm, recurrent, latent, feedforward, normed_attention  # noqa: F401
from . import gated_attention, linear_recurrent, parallel, token_input, rotary_attention, gated_average  # noqa: F401
from . import hyper_streams, differential_attention  # noqa: F401
