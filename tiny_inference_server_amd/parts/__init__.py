"""Parts that layers are put together from: norms, position encodings, mixers, feed-forwards,
block arrangements and stage inputs. Importing this package registers the built-in kinds."""
from .base import (ARRANGEMENTS, CONNECTIONS, FEED_FORWARDS, GATES, MIXERS, NORMS, POSITION_ENCODINGS, ROW_SHIFTS, STAGE_INPUTS,
                   TOKEN_INPUTS, Arrangement, CallContext, Tensors, build_part, expected_tensors, part_class, to_compute, to_gain)
from .spec import LayerCall, LayerSpec, ModelSpec, PagedKvNeed, PartSpec, StageSpec, StateNeed
from . import attention, block, feed_forward, hyper32, norm, parallel32, position, prenorm32, recurrent, stage_input, stream32  # noqa: F401  (registration)
