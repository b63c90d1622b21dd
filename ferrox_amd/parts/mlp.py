"""Dense gated feed-forward: down( act(gate x) * (up x) ), act = silu for this architecture
(ferrox-moe/src/lib.rs:655-658; dense layers: ferrox-models/src/decoder.rs:2902-2913).  The
activation is a parameter of the part and of the product's epilogue (`ops.ACTIVATIONS`)."""
from __future__ import annotations

import torch

from .. import debug, ops
from .base import FEED_FORWARDS, FeedForward, ParamSpec
from .linear import Linear, same_dtype


@FEED_FORWARDS.register("gated_mlp")
class GatedMLP(FeedForward):
    kernel_libraries = ("gemm",)
    TENSORS = {"gate": "gate_proj.weight", "up": "up_proj.weight", "down": "down_proj.weight"}

    def __init__(self, hidden_size: int, intermediate_size: int, activation: str = "silu", names: dict | None = None,
                 activation_params: tuple = (0.0, 0.0)):
        """`names`: what the checkpoint calls the three matrices, where that differs from `TENSORS`.
        `activation_params`: the numbers of an activation that has some (`ops.gemm`)."""
        if activation not in ops.ACTIVATIONS:
            raise ValueError(f"activation '{activation}' is not one of {sorted(ops.ACTIVATIONS)}")
        self.hidden_size, self.intermediate_size = int(hidden_size), int(intermediate_size)
        self.activation = activation
        self.activation_params = tuple(float(p) for p in activation_params)
        self.names = dict(self.TENSORS, **(names or {}))
        self.gate_up = self.down = None

    def param_specs(self):
        H, I, n = self.hidden_size, self.intermediate_size, self.names
        return {n["gate"]: ParamSpec((I, H)), n["up"]: ParamSpec((I, H)), n["down"]: ParamSpec((H, I))}

    def load(self, fetch):
        n = self.names
        self.gate_up = Linear(torch.cat(same_dtype([fetch(n["gate"]), fetch(n["up"])]), dim=0))
        self.down = Linear(fetch(n["down"]))

    def output(self, x):
        """The feed-forward's output as float32 [T, H], added to nothing."""
        return self.down(self._act(x), epilogue=ops.EPI_STORE_F32)

    def _act(self, x):
        return self.gate_up(x, epilogue=ops.EPI_GATED, activation=self.activation, activation_params=self.activation_params)

    takes_fresh = True       # forward(..., fresh=True): `residual` holds nothing yet, the output is stored into it

    def forward(self, x, ctx, residual, row_scale=None, fresh: bool = False) -> None:
        debug.region("mlp gate/up")
        act = self._act(x)
        debug.region("mlp down")
        if fresh and row_scale is None:
            self.down(act, epilogue=ops.EPI_STORE_F32, out=residual)
            return
        if fresh:
            ops.fill_u32(residual, 0)
        self.down(act, epilogue=ops.EPI_RESID, out=residual, row_scale=row_scale)


@FEED_FORWARDS.register("mlp")
class UngatedMLP(FeedForward):
    """down( act(up x) ): a feed-forward without a gate; the activation is the first product's epilogue
    (`ops.STORED_ACTIVATIONS`), e.g. "relu2", the square of relu."""
    kernel_libraries = ("gemm",)
    TENSORS = {"up": "up_proj.weight", "down": "down_proj.weight"}
    takes_fresh = True

    def __init__(self, hidden_size: int, intermediate_size: int, activation: str = "relu2", names: dict | None = None):
        if activation is None or activation not in ops.STORED_ACTIVATIONS:
            raise ValueError(f"activation '{activation}' is not one of {sorted(k for k in ops.STORED_ACTIVATIONS if k)}")
        self.hidden_size, self.intermediate_size, self.activation = int(hidden_size), int(intermediate_size), activation
        self.names = dict(self.TENSORS, **(names or {}))
        self.up = self.down = None

    def param_specs(self):
        return {self.names["up"]: ParamSpec((self.intermediate_size, self.hidden_size)),
                self.names["down"]: ParamSpec((self.hidden_size, self.intermediate_size))}

    def load(self, fetch):
        self.up, self.down = Linear(fetch(self.names["up"])), Linear(fetch(self.names["down"]))

    def forward(self, x, ctx, residual, fresh: bool = False) -> None:
        debug.region("mlp up")
        act = self.up(x, store_activation=self.activation)
        debug.region("mlp down")
        self.down(act, epilogue=ops.EPI_STORE_F32 if fresh else ops.EPI_RESID, out=residual)


@FEED_FORWARDS.register("swiglu")
class SwiGLU(GatedMLP):
    """The gated feed-forward with silu, under the name this architecture's description uses."""

    def __init__(self, hidden_size: int, intermediate_size: int):
        super().__init__(hidden_size, intermediate_size, "silu")
