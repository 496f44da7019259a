"""Parts of a layer, chosen by kind from registries.  Importing this package registers the built-in ones."""
from .base import (CacheNeed, ParamSpec, Part, StateNeed, build_part, known_parts, register_part,
                   unregister_part)
from . import (attention, block, delta, differential, ffn, latent, lightning, memory, norm, parallel, rope, shift, side,  # noqa: F401
               ssd)  # noqa: F401
