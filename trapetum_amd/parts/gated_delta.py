"""The gated delta rule: a matrix memory per head that decays and unlearns a key's old value before it writes the new one.

From the mixer's input x: q = W_q x, k = W_k x (kv_heads x key_dim), v = W_v x (heads x value_dim), each through a short
causal convolution over time on every channel (zeros before the sequence, no bias) and SiLU; q and k become unit vectors
per head, x / sqrt(sum x^2 + 1e-6), and q is multiplied by key_dim^(-1/2).  Head h uses q and k of kv head
h // (heads / kv_heads).  Per head and token, with beta = sigmoid(W_b x) and g = exp(-exp(A_log) softplus(W_a x + dt_bias)),

    S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q          (S is key_dim x value_dim, zero before the sequence)

and every head's o is divided by its root mean square, multiplied by a gain that the heads share and by silu(W_g x),
and projected back.  Decays, steps, unit norms, S, o and its norm are float32; the projections (one product for all
six) and the convolutions' outputs are in the activation dtype.  What a sequence keeps between steps is S and the
convolutions' last taps - 1 inputs, float32 states by name; there is nothing per token.
"""
from ..cache.store import StateSpec
from ..models.spec import TensorSpec
from ..registry import register_part
from .base import Mixer


class GatedDelta(Mixer):
    output_dtype = None          # a mixer that holds this one may ask for its last product in another dtype

    def __init__(self, hidden_size, num_heads, num_kv_heads, key_dim, value_dim, conv_taps, norm_eps,
                 tensors=("q", "k", "v", "g", "b", "a", "o", "norm", "A_log", "dt_bias"), conv_suffix=".conv"):
        """tensors: the local names of the six projections, W_o, the shared gain and the two vectors of the decay;
        a convolution is named like its projection with conv_suffix."""
        self.hidden_size, self.num_heads, self.num_kv_heads = int(hidden_size), int(num_heads), int(num_kv_heads)
        self.key_dim, self.value_dim, self.taps = int(key_dim), int(value_dim), int(conv_taps)
        self.norm_eps = float(norm_eps)
        if self.num_heads % self.num_kv_heads:
            raise ValueError(f"{num_heads} heads are no multiple of {num_kv_heads} kv heads")
        if self.taps < 1:
            raise ValueError(f"a convolution needs at least one tap, found {conv_taps}")
        self.names = dict(zip(("q", "k", "v", "g", "b", "a", "o", "norm", "a_log", "dt_bias"), tensors))
        self.conv_suffix = conv_suffix

    @property
    def conv_channels(self):
        return 2 * self.num_kv_heads * self.key_dim + self.num_heads * self.value_dim

    def tensor_specs(self):
        n, d, H = self.names, self.hidden_size, self.num_heads
        qk, vv = self.num_kv_heads * self.key_dim, H * self.value_dim
        specs = {n["q"]: TensorSpec((qk, d)), n["k"]: TensorSpec((qk, d)), n["v"]: TensorSpec((vv, d)), n["g"]: TensorSpec((vv, d)),
                 n["b"]: TensorSpec((H, d)), n["a"]: TensorSpec((H, d)), n["o"]: TensorSpec((d, vv)),
                 n["norm"]: TensorSpec((self.value_dim,), init="gain"),
                 n["a_log"]: TensorSpec((H,), init="norm"), n["dt_bias"]: TensorSpec((H,), init="norm")}
        for s, channels in (("q", qk), ("k", qk), ("v", vv)):
            specs[n[s] + self.conv_suffix] = TensorSpec((channels, self.taps), init="conv")
        return specs

    def state_specs(self):
        specs = {"memory": StateSpec((self.num_heads, self.key_dim, self.value_dim), "float32")}
        if self.taps > 1:
            specs["conv"] = StateSpec((self.taps - 1, self.conv_channels), "float32")
        return specs

    def bind(self, tensors, rt):
        import torch
        self.rt = rt
        n = self.names
        w = torch.cat([tensors[n[s]] for s in ("q", "k", "v", "g", "b", "a")], dim=0)
        spare = -w.shape[0] % 8                  # zero rows: a row of the product is whole 16-byte pieces
        if spare:
            w = torch.cat([w, w.new_zeros((spare, w.shape[1]))], dim=0)
        self.w_in = rt.matrix(w.contiguous())
        self.conv_t = torch.cat([tensors[n[s] + self.conv_suffix] for s in ("q", "k", "v")], dim=0).float().t().contiguous()     # [taps, channels]
        self.a_log = tensors[n["a_log"]].float().contiguous()
        self.dt_bias = tensors[n["dt_bias"]].float().contiguous()
        self.norm_gain = tensors[n["norm"]].float().repeat(self.num_heads).contiguous()
        self.w_o = rt.matrix(tensors[n["o"]])

    def forward(self, ctx, x, site):
        ops, H = ctx.ops, self.num_heads
        qk, vv, ch = self.num_kv_heads * self.key_dim, H * self.value_dim, self.conv_channels
        state = self.state(ctx, "conv") if self.taps > 1 else None
        if ctx.mode == "decode":                 # the product may stay in K slices until the convolution's launch
            p = u = ops.conv_step(ops.linear(x, self.w_in, ctx.dtype, defer=True), self.conv_t, state, ctx.slot_ids, ctx.dtype, activation="silu")
        else:
            p = ops.linear(x, self.w_in, ctx.dtype)                                               # [M, q | k | v | g | b | a]
            u = ops.conv_act(p[:, :ch], self.conv_t, None, state, ctx.slot_ids, ctx.cu_rows, ctx.row_seq, activation="silu")
        y = ops.delta_scan(u[:, :qk], u[:, qk:2 * qk], u[:, 2 * qk:ch], p[:, ch + vv:ch + vv + H], p[:, ch + vv + H:ch + vv + 2 * H],
                           self.a_log, self.dt_bias, self.state(ctx, "memory"), ctx.slot_ids, ctx.cu_rows, ctx.max_count, H,
                           self.num_kv_heads, self.key_dim, self.value_dim, self.key_dim ** -0.5)
        y = ops.head_norm_gate(y, self.norm_gain, p[:, ch:ch + vv], self.norm_eps, H, "silu", ctx.dtype)
        if self.output_dtype is not None:
            return ops.linear(y, self.w_o, self.output_dtype)
        return ops.linear(y, self.w_o, ctx.dtype, defer=True)


register_part("mixer", "gated_delta", GatedDelta)
