"""Python driver of the Sopanex host runtime (libpegainfer_qwen3.so, include/pegainfer_sopanex.h).

Sopanex lists its layers one by one in config.json.  A layer's mixer is a pair that reads one input side by side: softmax attention whose
values are its unrotated keys (a sink and a gate per head, long-context rotation) and gated linear attention with a decay per key
channel; its feed-forward is a routed one with identity experts and a gated shared expert, or none.  Every sublayer is normed before and
after.  The embedding may add a row chosen by the previous and the current token, so a request carries its last token.
A request holds cache pages AND a region of recurrent state; both are handed out again when it is dropped.
"""
from .step_engine import DTYPES, StepEngine  # noqa: F401


class SopanexEngine(StepEngine):
    architecture = "Sopanex"
    prefix = "pegainfer_sopanex_"

    def state_floats(self):
        """fp32 values of recurrent state one request holds"""
        return int(self._fn("state_floats")(self.h))
