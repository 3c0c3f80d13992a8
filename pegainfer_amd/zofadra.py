"""Python driver of the Zofadra host runtime (libpegainfer_qwen3.so, include/pegainfer_zofadra.h).

Zofadra lists its layers one by one in config.json and keeps several residual streams: a sublayer reads a learned weighted sum of
them through a layer norm, and its output joins every stream while a learned matrix mixes them.  Mixers: "latent_attention"
(queries through a normed latent, one cached latent and one rotated key part per token; a layer may read the latents of another),
"attention" (whole-row q / k norms, a sliding window, a bias falling linearly with the distance) and "lightning" (linear attention
with a constant decay per head).  Feed-forward: gelu(gate) * up, or none.
A request holds cache pages AND a region of recurrent state; both are handed out again when it is dropped.
"""
from .step_engine import DTYPES, StepEngine  # noqa: F401


class ZofadraEngine(StepEngine):
    architecture = "Zofadra"
    prefix = "pegainfer_zofadra_"

    def state_floats(self):
        """fp32 values of recurrent state one request holds"""
        return int(self._fn("state_floats")(self.h))
