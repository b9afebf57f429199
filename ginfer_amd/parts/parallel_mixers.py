"""Several mixers side by side on the same input, their results added with a factor each."""
import torch

from ..kernels import ops
from .base import Part
from .linear import linear
from .registry import register_mixer


@register_mixer("parallel_sum")
class ParallelSum(Part):
    """out = sum_i scale_i * mixer_i(x): `branches` are mixers of any kind (the model builds them from their `PartSpec`s),
    `names` the prefixes of their tensors inside this part, `scales` a factor each.  What a run keeps per request is the
    branches' caches one after the other (every branch gets its own share of the list of views, in the shape it
    declared).  The sum is taken in 32-bit.

    Where both branches can leave their products to others (`shares_products`: `hand_over_products`, `core`, `result_width`),
    there is ONE product for both projections (they read the same rows) and one for both outputs over the results side by side,
    which adds the branches up in its 32-bit accumulators; the factors are put into the results before they are rounded."""

    def __init__(self, branches, names, scales, dtype, device):
        self.branches, self.names, self.scales = list(branches), [str(n) for n in names], [float(s) for s in scales]
        if not (len(self.branches) == len(self.names) == len(self.scales) == 2):
            raise ValueError("two mixers side by side, each with a name and a factor; got %d, %d, %d"
                             % (len(self.branches), len(self.names), len(self.scales)))
        self.dtype, self.device = dtype, device
        self.w_in = self.w_out = None
        self.capturable = all(getattr(b, "capturable", False) for b in self.branches)

    def _shares(self):
        """Per branch: (its spec as it declared it, how many places of the common list it takes)."""
        out = []
        for b in self.branches:
            spec = b.cache_spec()
            out.append((spec, len(spec) if isinstance(spec, (list, tuple)) else 1))
        return out

    def cache_spec(self):
        specs = []
        for spec, _ in self._shares():
            specs += list(spec) if isinstance(spec, (list, tuple)) else [spec]
        return specs

    def weight_specs(self):
        return {n + "." + local: ws for n, b in zip(self.names, self.branches) for local, ws in b.weight_specs().items()}

    def bind_weights(self, tensors):
        for n, b in zip(self.names, self.branches):
            b.bind_weights({local: tensors[n + "." + local] for local in b.weight_specs()})
        if all(getattr(b, "shares_products", False) for b in self.branches):
            self._take_products()

    def _take_products(self):
        handed = [b.hand_over_products() for b in self.branches]
        self._columns, at = [], 0
        for w_in, _ in handed:
            self._columns.append((at, at + w_in.shape[0]))
            at += w_in.shape[0]
        self.w_in = torch.cat([h[0] for h in handed], dim=0).contiguous()
        widths = [b.result_width for b in self.branches]
        self._results = [(0, widths[0]), (widths[0], widths[0] + widths[1])]
        self._padding = -sum(widths) % 8             # the products take rows in steps of 8 elements
        outs = [h[1] for h in handed]
        if self._padding:
            outs.append(torch.zeros((outs[0].shape[0], self._padding), dtype=outs[0].dtype, device=outs[0].device))
        self.w_out = torch.cat(outs, dim=1).contiguous()

    def kernel_modules(self):
        mods = ["activation", "gemm"] + (["gemm_skinny"] if self.dtype == torch.bfloat16 else [])
        for b in self.branches:
            mods += [m for m in b.kernel_modules() if m not in mods]
        return mods

    def forward(self, x, step, cache):
        if self.w_in is not None:
            return self._forward_shared(x, step, cache)
        results, at = [], 0
        for b, (spec, n) in zip(self.branches, self._shares()):
            share = cache[at:at + n]
            at += n
            # (a result may be the 32-bit partial sums of a product whose K was split: the sum's kernel adds them up)
            results.append(b.forward(x, step, share if isinstance(spec, (list, tuple)) else share[0]))
        return ops.scaled_sum(results[0], results[1], self.scales[0], self.scales[1], self.dtype)

    def _forward_shared(self, x, step, cache):
        proj = linear(x, self.w_in, None, out_dtype=torch.float32)
        make = torch.zeros if self._padding else torch.empty
        both = make((x.shape[0], self.w_out.shape[1]), dtype=self.dtype, device=x.device)
        at = 0
        for b, (spec, n), (c0, c1), (r0, r1), scale in zip(self.branches, self._shares(), self._columns, self._results, self.scales):
            share = cache[at:at + n]
            at += n
            b.core(proj[:, c0:c1], step, share if isinstance(spec, (list, tuple)) else share[0], out=both[:, r0:r1], out_scale=scale)
        return linear(both, self.w_out, parts_ok=True)
