"""MI355X-native A81W41 quantized linear layer (Q8_1-style activations x Q4_1-style
int4 weights in the 8-column x 64-K interleaved block packing).

The compute path is the HIP libraries ``csrc/liba81w41*.so`` behind a C ABI
(``include/a81w41.h``, ``include/a81w41_model.h``); this package is a thin ctypes
binding, the model registry and the deterministic input generator.  There is no CPU fallback: every op raises if
the library is missing.
"""
from . import synth  # noqa: F401
from . import capi  # noqa: F401
from . import models  # noqa: F401
from . import ops  # noqa: F401
from .models import Model  # noqa: F401
from .ops import Linear, Qwen3Model  # noqa: F401
