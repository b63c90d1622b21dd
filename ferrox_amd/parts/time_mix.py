"""`time_mix`: a linear recurrence with a decay per token and key channel and a bonus for the current token, read by
mixes of every token with the one before it; a state of fixed size per request, no pages.  With h the mixer's input
row, h' the row of the token before (zeros before the first), heads of D key and D value channels:
    x_s = h + (h' - h) * mu_s                                                 one mix per reader s in r, k, v, g, w
    r, k, v = W_r x_r, W_k x_k, W_v x_v                                       heads x D
    d = exp(-exp(W_w2 tanh(W_w1 x_w) + w0))                                   a decay per head and key channel
    o = (S + diag(u) k v^T)^T r;   S <- diag(d) S + k v^T                     S: [D, D] per head, from zero
    y = W_o (o / rms(o) per head * w_norm * silu(W_g x_g))                    w_norm: one weight per head and channel
S and the last h are carried in the request's slot; everything behind the projections is float32.
"""
from __future__ import annotations

import torch

from .. import debug, ops
from .base import MIXERS, Mixer, ParamSpec
from .gated_linear import _add_out, longest_portion
from .linear import Linear, matmul, same_dtype
from .recurrent import sequence_starts

READERS = ("r", "k", "v", "g")      # the four projections of one shape, in the order of their planes; then the decay's
_groups: dict = {}


def reader_groups(device, n_tokens: int, n_groups: int, unsorted: bool):
    """Row -> group maps of a product of n_groups matrices with n_tokens rows each, the rows of group j being
    [j * n_tokens, (j + 1) * n_tokens): the group of every row (`unsorted`), or the groups' first rows.  Kept for the life
    of the process: recorded steps hold the addresses."""
    key = (torch.device(device), n_tokens, n_groups, unsorted)
    if key not in _groups:
        groups = torch.arange(n_groups + (0 if unsorted else 1), dtype=torch.int32)
        _groups[key] = (groups.repeat_interleave(n_tokens) if unsorted else groups * n_tokens).to(device)
        if len(_groups) > 4096:       # (prompt portions of many lengths: the oldest tables go; recorded sizes are few)
            _groups.pop(next(iter(_groups)))
    return _groups[key]


@MIXERS.register("time_mix")
class TimeMix(Mixer):
    kernel_libraries = ("elementwise", "gemm", "recurrent")
    graph_safe = True
    takes_fresh = True
    TENSORS = {"r": "r", "k": "k", "v": "v", "gate": "g", "mix": "mu.{}", "decay_in": "w1", "decay_out": "w2", "decay_base": "w0",
               "bonus": "u", "norm": "norm", "o": "o"}

    def __init__(self, hidden_size: int, n_heads: int, head_dim: int, norm_eps: float, decay_rank: int, names: dict | None = None):
        """`decay_rank`: the inner size of the decay's low-rank projection.  `names["mix"]` is a pattern that the
        reader's letter goes into."""
        self.hidden_size, self.n_heads, self.head_dim = int(hidden_size), int(n_heads), int(head_dim)
        if not 1 <= self.head_dim <= 256:
            raise ValueError(f"head_dim {head_dim}: the recurrence kernel holds up to 256 key channels a head")
        self.norm_eps, self.decay_rank = float(norm_eps), int(decay_rank)
        if self.decay_rank < 1:
            raise ValueError(f"a decay projection of inner size {decay_rank}")
        self.names = dict(self.TENSORS, **(names or {}))
        self.inner = self.n_heads * self.head_dim
        self.w_in = self.w_decay = self.mu = self.decay_out_t = self.decay_base = self.bonus = self.norm_w = self.o_proj = None

    def param_specs(self):
        W, I, n = self.hidden_size, self.inner, self.names
        specs = {n[x]: ParamSpec((I, W)) for x in ("r", "k", "v", "gate")}
        specs.update({n["mix"].format(s): ParamSpec((W,)) for s in READERS + ("w",)})
        specs.update({n["decay_in"]: ParamSpec((self.decay_rank, W)), n["decay_out"]: ParamSpec((I, self.decay_rank)),
                      n["decay_base"]: ParamSpec((I,)), n["bonus"]: ParamSpec((self.n_heads, self.head_dim)),
                      n["norm"]: ParamSpec((I,), init="ones"), n["o"]: ParamSpec((W, I))})
        return specs

    def load(self, fetch):
        n = self.names
        # the four matrices of one shape as the groups of one product
        self.w_in = torch.stack(same_dtype([fetch(n[x]) for x in ("r", "k", "v", "gate")])).contiguous()
        self.w_decay = fetch(n["decay_in"]).contiguous()
        self.mu = torch.stack([fetch(n["mix"].format(s)).float() for s in READERS + ("w",)]).contiguous()
        # what feeds the recurrence stays float32 (the second half of the decay's projection transposed, a column a thread)
        self.decay_out_t = fetch(n["decay_out"]).float().t().contiguous()
        self.decay_base = fetch(n["decay_base"]).float().contiguous()
        self.bonus = fetch(n["bonus"]).float().contiguous()
        self.norm_w = fetch(n["norm"]).float().contiguous()
        self.o_proj = Linear(fetch(n["o"]))

    def state_shapes(self) -> dict:
        return {"S": ((self.n_heads, self.head_dim, self.head_dim), torch.float32),      # transposed: [head][value][key]
                "last": ((self.hidden_size,), torch.float32)}

    def read(self, mixes):
        """The four projections of their mixes [>= 4, T, hidden], float32 [4, T, inner]."""
        T, W = mixes.shape[1], self.hidden_size
        rows = mixes[:4].reshape(4 * T, W)
        if rows.dtype != self.w_in.dtype:            # (a checkpoint that stores these matrices in float32)
            rows = ops.cast(rows, self.w_in.dtype)
        out = torch.empty((4 * T, self.inner), dtype=torch.float32, device=rows.device)
        if rows.dtype == torch.bfloat16 and 4 * T <= 64 and W % 8 == 0 and rows.data_ptr() % 16 == 0 and self.w_in.data_ptr() % 16 == 0:
            ops.gemm(rows, self.w_in, epilogue=ops.EPI_STORE_F32, pair_ids=reader_groups(rows.device, T, 4, True), out=out)
        else:
            ops.gemm(rows, self.w_in, epilogue=ops.EPI_STORE_F32, expert_offsets=reader_groups(rows.device, T, 4, False), out=out)
        return out.view(4, T, self.inner)

    def forward(self, x, ctx, cache, residual, out_scale: float | None = None, fresh: bool = False) -> None:
        H, D = self.n_heads, self.head_dim
        starts = sequence_starts(ctx)
        debug.region("token shift")
        mixes = ops.token_shift(x, self.mu, cache.state["last"], ctx.token_seq, starts, ctx.slot_ids)
        debug.region("time mix in")
        r, k, v, gate = self.read(mixes)
        low = matmul(mixes[4], self.w_decay, epilogue=ops.EPI_STORE_F32)
        debug.region("time mix decay")
        keep = ops.lowrank_decay(low, self.decay_out_t, self.decay_base)
        debug.region("linear recurrence")
        o = ops.channel_outer(r, k, v, keep, self.bonus, cache.state["S"], starts, ctx.slot_ids, ctx.n_seqs, H, D, D,
                              longest=longest_portion(ctx))
        debug.region("time mix out")
        y = ops.gated_head_norm(o, gate, self.norm_w, self.norm_eps, H, D, ctx.act_dtype, gate_activation="silu")
        _add_out(self.o_proj, y, ctx, residual, out_scale, fresh)
