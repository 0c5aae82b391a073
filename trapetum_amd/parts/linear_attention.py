"""Linear attention whose memory decays by a constant per head (lightning attention).

From the mixer's input x: q = silu(W_q x), k = silu(W_k x) (heads x key_dim), v = silu(W_v x) (heads x value_dim).  Per head
and token, with the head's decay g, a constant of the model,

    S <- g S + v k^T,   o = S q                     (S is value_dim x key_dim, zero before the sequence; no other scale)

and the concatenated heads' o is divided, whole, by its root mean square, multiplied by a gain and by sigmoid(W_g x), and
projected back.  S, the decays, o and its norm are float32; q, k, v and the gate come from one product whose first columns
pass SiLU before they are rounded to the activation dtype.  What a sequence keeps between steps is S, a float32 state by
name; there is nothing per token, so a step costs the same at any length.
"""
from ..cache.store import StateSpec
from ..models.spec import TensorSpec
from ..registry import register_part
from .base import Mixer


class LinearAttention(Mixer):
    output_dtype = None          # a mixer that holds this one may ask for its last product in another dtype

    def __init__(self, hidden_size, num_heads, key_dim, value_dim, decay, norm_eps, tensors=("q", "k", "v", "g", "o", "norm")):
        """decay: a number per head, at least 0 and at most 1.  tensors: the local names of the five matrices and the gain."""
        self.hidden_size, self.num_heads = int(hidden_size), int(num_heads)
        self.key_dim, self.value_dim = int(key_dim), int(value_dim)
        self.decay_values = tuple(float(d) for d in decay)
        self.norm_eps = float(norm_eps)
        if len(self.decay_values) != self.num_heads:
            raise ValueError(f"{len(self.decay_values)} decays for {num_heads} heads")
        if not all(0.0 <= d <= 1.0 for d in self.decay_values):
            raise ValueError("a decay lies between 0 and 1")
        self.names = dict(zip(("q", "k", "v", "g", "o", "norm"), tensors))

    def tensor_specs(self):
        n, d, H = self.names, self.hidden_size, self.num_heads
        qk, vv = H * self.key_dim, H * self.value_dim
        return {n["q"]: TensorSpec((qk, d)), n["k"]: TensorSpec((qk, d)), n["v"]: TensorSpec((vv, d)), n["g"]: TensorSpec((vv, d)),
                n["o"]: TensorSpec((d, vv)), n["norm"]: TensorSpec((vv,), init="gain")}

    def state_specs(self):
        return {"memory": StateSpec((self.num_heads, self.value_dim, self.key_dim), "float32")}

    def bind(self, tensors, rt):
        import torch
        self.rt = rt
        n = self.names
        w = torch.cat([tensors[n[s]] for s in ("q", "k", "v", "g")], dim=0)
        spare = -w.shape[0] % 8                  # zero rows: a row of the product is whole 16-byte pieces
        if spare:
            w = torch.cat([w, w.new_zeros((spare, w.shape[1]))], dim=0)
        self.w_in = rt.matrix(w.contiguous())
        self.decay = torch.tensor(self.decay_values, dtype=torch.float32, device=rt.device)
        self.norm_gain = tensors[n["norm"]].float().contiguous()
        self.w_o = rt.matrix(tensors[n["o"]])

    def forward(self, ctx, x, site):
        ops, H = ctx.ops, self.num_heads
        qk, vv = H * self.key_dim, H * self.value_dim
        u = ops.linear_act(x, self.w_in, ctx.dtype, "silu", columns=2 * qk + vv)                     # [M, q | k | v | g]
        y = ops.linear_scan(u[:, :qk], u[:, qk:2 * qk], u[:, 2 * qk:2 * qk + vv], self.decay, self.state(ctx, "memory"),
                            ctx.slot_ids, ctx.cu_rows, ctx.max_count, H, self.key_dim, self.value_dim)
        y = ops.head_norm_gate(y, self.norm_gain, u[:, 2 * qk + vv:2 * qk + 2 * vv], self.norm_eps, 1, "sigmoid", ctx.dtype)
        if self.output_dtype is not None:
            return ops.linear(y, self.w_o, self.output_dtype)
        return ops.linear(y, self.w_o, ctx.dtype, defer=True)


register_part("mixer", "linear_attention", LinearAttention)
