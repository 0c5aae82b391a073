"""How a layer's parts are arranged around the residual stream.

sandwich  x += post_mixer_norm(mixer(pre_mixer_norm(x)));
          x += post_ff_norm(ff(pre_ff_norm(x)))          (runtime/src/lib.rs:4527-4540)
pre_norm  x += mixer(pre_mixer_norm(x));  x += ff(pre_ff_norm(x)); the feed-forward may be absent
          (the reference's other layer type, runtime/src/lib.rs:721-730).  With `token_shift` the mixer reads
          h + (h' - h) * w instead of h = pre_mixer_norm(x), h' being the h of the token before (zeros before the
          sequence) and w a vector of the layer; the last token's h is a state of the sequence.  With `residual_scale` m
          a sub-layer's output is multiplied by m before it is added.
post_norm x += post_mixer_norm(mixer(c1(x)));  x += post_ff_norm(ff(c2(x))): no norm in front of a sub-layer; c1
          and c2 are what it reads of the stream, the stream itself or (input_conv) the stream through a short
          causal convolution whose last rows are a state of the sequence.  The feed-forward may be absent.
parallel  x += mixer(n(x)) + ff(n(x)): one norm, and both sub-layers read its output; the feed-forward may be absent.

The stream is fp32 and the sum is formed in fp32 (the reference adds in fp32 and
stores fp16: runtime/cuda/codebook_gemv.cu:539-542).  Where a norm of a sub-layer's
output is followed by the add and by the next norm, one kernel does all three; that
includes the first norm of the block that runs next (`next_norm`), whose result the
next block receives as `normed`.  What a model adds to the stream between two layers (`NormAfterAdd`) is added in
that kernel too.
"""
from ..registry import register_part
from .base import Block


def add_then_norm(ctx, stream, rows, post, nxt, scale=1.0):
    """stream += scale * post(rows) (or rows); returns nxt(stream) (or None).  One kernel when both norms
    expose an RMS gain, else the norms' own forward around a plain add."""
    pair = isinstance(rows, ctx.ops.WeightedRows)
    if post is None and (pair or scale != 1.0):          # constants on the rows: the kernel that adds two operands takes them
        a, wa, b, wb = (rows.a, rows.wa, rows.b, rows.wb) if pair else (rows, 1.0, None, 1.0)
        return join_then_norm(ctx, stream, a, b, nxt, wa * scale, wb * scale)
    if scale != 1.0:
        raise ValueError("a residual scale goes with blocks that do not norm a sub-layer's output")
    if pair:
        rows = ctx.ops.rows(rows, ctx.dtype)
    if isinstance(nxt, NormAfterAdd):
        if post is None:
            return join_then_norm(ctx, stream, rows, None, nxt)
        add_then_norm(ctx, stream, rows, post, None)
        return nxt.forward(ctx, stream)
    fusable = all(n is None or n.gain is not None for n in (post, nxt))
    groups = {getattr(n, "groups", 1) for n in (post, nxt) if n is not None}      # one kernel cuts both norms alike
    if fusable and len(groups) <= 1:
        return ctx.ops.add_rms_norm(stream, rows,
                                    post.gain if post else None, post.eps if post else 0.0,
                                    nxt.gain if nxt else None, nxt.eps if nxt else 0.0,
                                    getattr(nxt, "reader_dtype", None) or ctx.dtype,       # a reader may ask for float32 rows
                                    groups=groups.pop() if groups else 1)
    rows = ctx.ops.rows(rows, ctx.dtype)
    if post is not None:
        rows = post.forward(ctx, rows)
    ctx.ops.add_rms_norm(stream, rows, None, 0.0, None, 0.0, ctx.dtype)
    return nxt.forward(ctx, stream, getattr(nxt, "reader_dtype", None)) if nxt is not None else None


class NormAfterAdd:
    """A block's first norm with what the model adds to the stream before that block: `added` is a StreamAdd part."""

    def __init__(self, norm, added):
        self.norm, self.added = norm, added                # norm None: the add alone
        self.gain = norm.gain if norm is not None else None

    def forward(self, ctx, stream, out_dtype=None):
        return join_then_norm(ctx, stream, None, None, self)


def join_then_norm(ctx, stream, a, b, nxt, wa=1.0, wb=1.0):
    """stream += wa a + wb b (either may be None) and what `nxt` does to the stream before its norm; returns its norm of the
    stream (or None)."""
    norm = nxt.norm if isinstance(nxt, NormAfterAdd) else nxt
    plain = norm is None or (norm.gain is not None and getattr(norm, "groups", 1) == 1)
    dtype = getattr(norm, "reader_dtype", None) or ctx.dtype
    gain, eps = (norm.gain, norm.eps) if plain and norm is not None else (None, 0.0)
    if isinstance(nxt, NormAfterAdd) and nxt.added.replaces:
        out = nxt.added.forward(ctx, stream, a, b, wa, wb, gain, eps, dtype)
    else:
        vec, origin = nxt.added.operands(ctx) if isinstance(nxt, NormAfterAdd) else (None, None)
        out = ctx.ops.join_rms_norm(stream, a, b, gain, eps, dtype, vec=vec, origin=origin, wa=wa, wb=wb)
    return out if plain else norm.forward(ctx, stream, getattr(norm, "reader_dtype", None))


class SandwichBlock(Block):
    def __init__(self, mixer, feed_forward, make_norm):
        self.mixer = mixer
        self.feed_forward = feed_forward                 # None: the layer is its mixer, with the norms around it
        sites = self.norm_sites() if feed_forward is not None else self.norm_sites()[:2]
        self.norms = {name: make_norm(name) for name in sites}

    @classmethod
    def norm_sites(cls):
        return ("pre_mixer_norm", "post_mixer_norm", "pre_ff_norm", "post_ff_norm")

    def entry_norm(self):
        return self.norms["pre_mixer_norm"]

    def forward(self, ctx, stream, site, normed=None, next_norm=None):
        n = self.norms
        x = normed if normed is not None else n["pre_mixer_norm"].forward(ctx, stream)
        ctx.dump("mixer_in", x)
        a = self.mixer.forward(ctx, x, site)
        ctx.dump("mixer_out", a)
        if self.feed_forward is None:
            normed_next = add_then_norm(ctx, stream, a, n["post_mixer_norm"], next_norm)
            ctx.dump("layer_out", stream)
            return stream, normed_next
        x = add_then_norm(ctx, stream, a, n["post_mixer_norm"], n["pre_ff_norm"])
        ctx.dump("after_mixer", stream)
        m = self.feed_forward.forward(ctx, x)
        ctx.dump("ff_out", m)
        normed_next = add_then_norm(ctx, stream, m, n["post_ff_norm"], next_norm)
        ctx.dump("layer_out", stream)
        return stream, normed_next


class PreNormBlock(Block):
    def __init__(self, mixer, feed_forward, make_norm, token_shift=None, residual_scale=1.0):
        """token_shift: the local name of the mixing vector [hidden] (None: the mixer reads the normed rows as they are).
        residual_scale: the constant a sub-layer's output is multiplied by."""
        self.residual_scale = float(residual_scale)
        self.mixer = mixer
        self.feed_forward = feed_forward                 # None: the layer is its mixer behind its norm
        sites = self.norm_sites() if feed_forward is not None else self.norm_sites()[:1]
        self.norms = {name: make_norm(name) for name in sites}
        self.token_shift = token_shift
        if token_shift is not None:
            import torch
            # the mix is formed in float32 from float32 rows and rounded once; whoever applies this block's first norm
            # (the block itself, or the block before in the kernel of its last add) leaves the rows in float32
            self.norms["pre_mixer_norm"].reader_dtype = torch.float32

    @classmethod
    def norm_sites(cls):
        return ("pre_mixer_norm", "pre_ff_norm")

    def entry_norm(self):
        return self.norms["pre_mixer_norm"]

    def tensor_specs(self):
        if self.token_shift is None:
            return {}
        from ..models.spec import TensorSpec
        return {self.token_shift: TensorSpec((self.norms["pre_mixer_norm"].size,), init="norm")}

    def state_specs(self):
        if self.token_shift is None:
            return {}
        from ..cache.store import StateSpec
        return {"token_shift": StateSpec((self.norms["pre_mixer_norm"].size,), "float32")}

    def bind(self, tensors, rt):
        self.rt = rt
        if self.token_shift is not None:
            self.shift_weight = tensors[self.token_shift].float().reshape(1, -1).contiguous()

    def forward(self, ctx, stream, site, normed=None, next_norm=None):
        n = self.norms
        first = n["pre_mixer_norm"]
        x = normed if normed is not None else first.forward(ctx, stream, getattr(first, "reader_dtype", None))
        if self.token_shift is not None:
            x = ctx.ops.shift_mix(x, self.shift_weight, ctx.cache.entry_state(ctx.entry, "token_shift"), ctx.slot_ids, ctx.cu_rows,
                                  ctx.row_seq, one_row_each=ctx.mode == "decode", out_dtype=ctx.dtype)[0]
        ctx.dump("mixer_in", x)
        a = self.mixer.forward(ctx, x, site)
        ctx.dump("mixer_out", a)
        if self.feed_forward is None:
            normed_next = add_then_norm(ctx, stream, a, None, next_norm, self.residual_scale)
            ctx.dump("layer_out", stream)
            return stream, normed_next
        x = add_then_norm(ctx, stream, a, None, n["pre_ff_norm"], self.residual_scale)
        ctx.dump("after_mixer", stream)
        m = self.feed_forward.forward(ctx, x)
        ctx.dump("ff_out", m)
        normed_next = add_then_norm(ctx, stream, m, None, next_norm, self.residual_scale)
        ctx.dump("layer_out", stream)
        return stream, normed_next


class PostNormBlock(Block):
    def __init__(self, mixer, feed_forward, make_norm, input_conv=None):
        """input_conv: (registered conv, parameters) built once in front of each sub-layer, or None."""
        from ..registry import build_part
        self.mixer = mixer
        self.feed_forward = feed_forward
        sites = ("post_mixer_norm", "post_ff_norm") if feed_forward is not None else ("post_mixer_norm",)
        self.norms = {name: make_norm(name) for name in sites}
        self.convs = {}
        if input_conv is not None:
            for site in ("mixer_conv", "ff_conv")[:len(sites)]:
                self.convs[site] = build_part("conv", input_conv)

    @classmethod
    def norm_sites(cls):
        return ("post_mixer_norm", "post_ff_norm")

    def inner_parts(self):
        return dict(self.convs)

    def state_specs(self):
        return {site: c.state_spec() for site, c in self.convs.items() if c.state_spec() is not None}

    def _read(self, ctx, stream, site):
        conv = self.convs.get(site)
        if conv is None:
            return stream.to(ctx.dtype)
        state = ctx.cache.entry_state(ctx.entry, site) if conv.state_spec() is not None else None
        return conv.forward(ctx, stream, state)

    def forward(self, ctx, stream, site, normed=None, next_norm=None):
        n = self.norms
        x = self._read(ctx, stream, "mixer_conv")
        ctx.dump("mixer_in", x)
        a = self.mixer.forward(ctx, x, site)
        ctx.dump("mixer_out", a)
        if self.feed_forward is None:
            normed_next = add_then_norm(ctx, stream, a, n["post_mixer_norm"], next_norm)
            ctx.dump("layer_out", stream)
            return stream, normed_next
        add_then_norm(ctx, stream, a, n["post_mixer_norm"], None)
        ctx.dump("after_mixer", stream)
        x = self._read(ctx, stream, "ff_conv")
        m = self.feed_forward.forward(ctx, x)
        ctx.dump("ff_out", m)
        normed_next = add_then_norm(ctx, stream, m, n["post_ff_norm"], next_norm)
        ctx.dump("layer_out", stream)
        return stream, normed_next


class ParallelBlock(Block):
    def __init__(self, mixer, feed_forward, make_norm):
        super().__init__(mixer, feed_forward, make_norm)

    @classmethod
    def norm_sites(cls):
        return ("pre_norm",)

    def entry_norm(self):
        return self.norms["pre_norm"]

    def forward(self, ctx, stream, site, normed=None, next_norm=None):
        x = normed if normed is not None else self.norms["pre_norm"].forward(ctx, stream)
        ctx.dump("mixer_in", x)
        a = self.mixer.forward(ctx, x, site)
        ctx.dump("mixer_out", a)
        m = None
        if self.feed_forward is not None:
            m = self.feed_forward.forward(ctx, x)
            ctx.dump("ff_out", m)
        normed_next = join_then_norm(ctx, stream, a, m, next_norm)       # with what the model adds before the next layer
        ctx.dump("layer_out", stream)
        return stream, normed_next


register_part("block", "parallel", ParallelBlock)
register_part("block", "sandwich", SandwichBlock)
register_part("block", "post_norm", PostNormBlock)
register_part("block", "pre_norm", PreNormBlock)
