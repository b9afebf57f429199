"""Recurrent mixers with one decay per token and head, over 32-bit state per request: the gated delta rule and Mamba-2's
state-space recurrence.  Both put their channels through a short causal convolution over time."""
import torch

from ..kernels import ops
from ..weights.loader import WeightSpec
from .base import Part, StateSpec
from .linear import linear
from .registry import register_mixer


class _DeltaMixer(Part):
    """What the two share: one projection (left in 32-bit) of everything that reads x, the step over state and ring
    (ops.delta_recurrence), and one output product.  The state lies in the order in which the kernels read it, the
    convolution's inputs in a ring of `taps` rows."""

    capturable = True

    def __init__(self, hidden_size, num_heads, num_groups, key_dim, value_dim, taps, eps, dtype, device):
        self.hidden_size, self.nh, self.ng = int(hidden_size), int(num_heads), int(num_groups)
        self.dk, self.dv, self.taps, self.eps = int(key_dim), int(value_dim), int(taps), float(eps)
        if self.ng < 1 or self.nh % self.ng:
            raise ValueError("%d heads do not fall into %d equal groups" % (self.nh, self.ng))
        if not 0 < self.dk <= ops.DELTA_MAX_DIM or not 0 < self.dv <= ops.DELTA_MAX_VDIM:
            raise ValueError("heads of %d x %d are not supported: the recurrence's kernels take up to %d x %d"
                             % (self.dk, self.dv, ops.DELTA_MAX_DIM, ops.DELTA_MAX_VDIM))
        if not 1 <= self.taps <= ops.SHORT_CONV_MAX_TAPS:
            raise ValueError("the short convolution takes 1 to %d taps, got %r" % (ops.SHORT_CONV_MAX_TAPS, taps))
        self.dtype, self.device = dtype, device
        self.channels = 2 * self.ng * self.dk + self.nh * self.dv
        self.w_in = self.w_o = self.w_conv = self.b_conv = self.rate = self.dt_bias = self.skip = self.norm_weight = None

    def cache_spec(self):
        """[the recurrence's state, the ring of the convolution's inputs (None for one tap)]."""
        ring = StateSpec((self.taps, self.channels), torch.float32) if self.taps > 1 else None
        return [StateSpec(ops.delta_state_shape(self.nh, self.dk, self.dv), torch.float32), ring]

    def kernel_modules(self):
        return ["delta_scan", "decay_scan", "gemm"] + (["delta_chunk", "gemm_skinny"] if self.dtype == torch.bfloat16 else [])

    def _recurrence(self, proj, step, cache, **kw):
        state, ring = cache
        return ops.delta_recurrence(proj, self.w_conv, self.b_conv, self.rate, self.dt_bias, self.skip, None if ring is None else ring.state,
                                    state.state, state.slots, step, self.nh, self.ng, self.dk, self.dv, self.columns, chunked=self.dtype == torch.bfloat16, **kw)

    # (what `ParallelSum` needs to share the two products: see ConvAttention)
    @property
    def result_width(self):
        return self.nh * self.dv

    def hand_over_products(self):
        out = (self.w_in, self.w_o)
        self.w_in = self.w_o = None
        return out

    def forward(self, x, step, cache):
        o = self.core(linear(x, self.w_in, None, out_dtype=torch.float32), step, cache)
        return linear(o, self.w_o, parts_ok=True)


@register_mixer("gated_delta")
class GatedDeltaRule(_DeltaMixer):
    """q, k, v = silu(conv(W x)) (q and k of `num_groups` heads, shared by the heads of a group); q and k become unit vectors per
    head, z / sqrt(sum z^2 + unit_eps), q times key_dim^(-1/2); b = sigmoid(Wb x), a = exp(-exp(A_log) * softplus(Wa x + dt_bias))
    per head; S <- a S, u = b (v - S^T k), S <- S + k u^T, o = S^T q; per head o / rms(o) * norm * silu(Wg x); then Wo.
    Tensors: q, q.conv, k, k.conv, v, v.conv, g, b, a, A_log, dt_bias, norm, o."""

    shares_products = True

    def __init__(self, hidden_size, num_heads, num_kv_heads, key_dim, value_dim, taps, eps, dtype, device, unit_eps=1e-6):
        super().__init__(hidden_size, num_heads, num_kv_heads, key_dim, value_dim, taps, eps, dtype, device)
        self.unit_eps = float(unit_eps)
        k, v = self.ng * self.dk, self.nh * self.dv
        # the projection's rows: q | k | v | g | b | a
        self.columns = dict(conv=0, q=0, k=k, v=2 * k, gate=2 * k + v, b=2 * k + 2 * v, a=2 * k + 2 * v + self.nh)

    def weight_specs(self):
        H, k, v, n = self.hidden_size, self.ng * self.dk, self.nh * self.dv, self.nh
        specs = {"q": WeightSpec((k, H)), "k": WeightSpec((k, H)), "v": WeightSpec((v, H)), "g": WeightSpec((v, H)),
                 "b": WeightSpec((n, H)), "a": WeightSpec((n, H)), "o": WeightSpec((H, v)),
                 "A_log": WeightSpec((n,), std=1.0, keep_32bit=True), "dt_bias": WeightSpec((n,), std=1.0, keep_32bit=True),
                 "norm": WeightSpec((self.dv,), init="one_plus_normal", keep_32bit=True)}
        for name, rows in (("q", k), ("k", k), ("v", v)):
            specs[name + ".conv"] = WeightSpec((rows, self.taps), std=0.5, keep_32bit=True)
        return specs

    def bind_weights(self, t):
        self.w_in = torch.cat([t[n] for n in ("q", "k", "v", "g", "b", "a")], dim=0).contiguous()
        self.w_conv = torch.cat([t[n + ".conv"].float() for n in ("q", "k", "v")], dim=0).contiguous()
        self.rate = torch.exp(t["A_log"].float()).contiguous()
        self.dt_bias = t["dt_bias"].float().contiguous()
        self.norm_weight = t["norm"].float().contiguous()
        self.w_o = t["o"]

    def core(self, proj, step, cache, out=None, out_scale=1.0):
        return self._recurrence(proj, step, cache, delta=True, q_scale=self.dk ** -0.5, unit_eps=self.unit_eps, weight=self.norm_weight,
                                eps=self.eps, dtype=self.dtype, out=out, out_scale=out_scale)


@register_mixer("mamba2")
class Mamba2(_DeltaMixer):
    """[z | x | B | C | d] = Win h (inner = heads * value_dim columns for z and x, groups * state for B and C, one d a head); x, B and
    C go through conv + bias and silu; d <- softplus(d + dt_bias); per head (with its group's B and C) S <- exp(-exp(A_log) d) S +
    d B x^T, y = S^T C + D x; y * silu(z) is RMS-normed in `norm_groups` equal parts of the row, times `norm`; then Wo.
    Tensors: in, conv, conv.b, dt_bias, A_log, D, norm, o."""

    def __init__(self, hidden_size, num_heads, value_dim, state_size, groups, norm_groups, taps, eps, dtype, device):
        super().__init__(hidden_size, num_heads, groups, state_size, value_dim, taps, eps, dtype, device)
        inner, bc = self.nh * self.dv, self.ng * self.dk
        self.norm_groups = int(norm_groups)
        if self.norm_groups < 1 or inner % self.norm_groups:
            raise ValueError("a row of %d does not fall into %d equal parts" % (inner, self.norm_groups))
        # among the convolved channels x | B | C: the key is B, the query C
        self.columns = dict(gate=0, conv=inner, v=0, k=inner, q=inner + bc, a=2 * inner + 2 * bc, b=2 * inner + 2 * bc)

    def weight_specs(self):
        H, inner, n = self.hidden_size, self.nh * self.dv, self.nh
        return {"in": WeightSpec((inner + self.channels + n, H)), "conv": WeightSpec((self.channels, self.taps), std=0.5, keep_32bit=True),
                "conv.b": WeightSpec((self.channels,), std=0.1, keep_32bit=True), "dt_bias": WeightSpec((n,), std=1.0, keep_32bit=True),
                "A_log": WeightSpec((n,), std=1.0, keep_32bit=True), "D": WeightSpec((n,), init="one_plus_normal", keep_32bit=True),
                "norm": WeightSpec((inner,), init="one_plus_normal", keep_32bit=True), "o": WeightSpec((H, inner))}

    def bind_weights(self, t):
        self.w_in, self.w_o = t["in"], t["o"]
        self.w_conv, self.b_conv = t["conv"].float().contiguous(), t["conv.b"].float().contiguous()
        self.rate = torch.exp(t["A_log"].float()).contiguous()
        self.dt_bias, self.skip = t["dt_bias"].float().contiguous(), t["D"].float().contiguous()
        self.norm_weight = t["norm"].float().reshape(self.norm_groups, -1).contiguous()

    def core(self, proj, step, cache):
        y = self._recurrence(proj, step, cache, delta=False)
        return ops.head_norm_gate(y.view(y.shape[0], self.norm_groups, -1), self.norm_weight, self.eps, self.dtype)
