"""Time mixing with a matrix state whose decays depend on the token (the RWKV family), with a fixed-size state per request.

With ``h'`` the input of the token before (zeros before the first), each of r, k, v, g and w reads a mix of its own, ``h + (h' - h) * mu_s``.  ``r``,
``k`` (``heads x dim``) and ``v`` (``heads x vdim``) are products of their mixes; the decay is ``w = exp(-exp(w0 + W_w2 tanh(W_w1 mix_w)))`` per
head and key channel.  Head by head, with the bonus ``u`` for the current token only::

    o = (S + diag(u) k v^T)^T r;    S <- diag(w) S + k v^T

and the mixer's output is ``W_o (concat_heads(o / rms(o)) * w_norm * silu(W_g mix_g))``.  A request's slot holds the states of all heads and the
last token's input, in 32-bit, zero when the slot is handed out.

The mixer reads the 32-bit stream itself where its block hands it over (``reads_stream``): one kernel lets what is pending enter the
stream and makes the five mixes; the four equal products are one launch; the decays, their logarithms and the state are 32-bit under every
engine.  The recurrence runs token by token from where the state stands, so a portion of n tokens is n single steps by construction.
"""
from __future__ import annotations

import torch

from ..config.base import ConfigError
from ..kernels import ops
from .base import KEEP_COMPUTE, KEEP_FLOAT32, MIXERS, Mixer, StateNeed, Stream, WeightSpec, project_out, register_init_law

MIXES = ("r", "k", "v", "g", "w")


@register_init_law("share")
def _init_share(shape, gen, device, std):
    """Shares between 0 and 1 (how much of a mix is the token before)."""
    return torch.rand(shape, generator=gen, device=device, dtype=torch.float32)


@register_init_law("log_log_decay")
def _init_log_log_decay(shape, gen, device, std):
    """``w0`` of decays ``exp(-exp(w0))`` between about 0.4 and 0.998."""
    return torch.rand(shape, generator=gen, device=device, dtype=torch.float32) * 6.0 - 6.0


@MIXERS.register("wkv")
class WKV(Mixer):
    graph_safe = True
    reads_stream = True

    def __init__(self, spec, dtype, device):
        super().__init__(spec, dtype, device)
        if spec.dim > ops.DELTA_MAX_DIM:
            raise ConfigError(f"wkv: built for up to {ops.DELTA_MAX_DIM} key dimensions per head, not {spec.dim}")
        self.hidden, self.heads, self.dim, self.vdim = spec.hidden, spec.heads, spec.dim, spec.vdim
        self.k_width, self.v_width = spec.heads * spec.dim, spec.heads * spec.vdim
        self.state_floats = spec.heads * spec.dim * spec.vdim         # the heads' states; the last token's input follows
        self.mu = self.w_rk = self.w_vg = self.w_rkvg = self.w1 = self.w2t = self.w0 = self.bonus = self.w_norm = self.w_o = None

    def state_need(self):
        return StateNeed(shape=(self.state_floats + self.hidden,), dtype=torch.float32)

    def kernel_libraries(self):
        return ["recurrent"]

    def weight_specs(self):
        H, K, V, rank = self.hidden, self.k_width, self.v_width, int(self.spec.decay_rank)
        specs = {f"mu.{s}": WeightSpec((H,), keep=KEEP_FLOAT32, init="share") for s in MIXES}
        specs.update({
            "r": WeightSpec((K, H)), "k": WeightSpec((K, H)), "v": WeightSpec((V, H)), "g": WeightSpec((V, H)),
            "w1": WeightSpec((rank, H), free_axes=(0,)), "w2": WeightSpec((K, rank), keep=KEEP_FLOAT32, free_axes=(1,)),
            "w0": WeightSpec((K,), keep=KEEP_FLOAT32, init="log_log_decay"), "u": WeightSpec((self.heads, self.dim), keep=KEEP_FLOAT32),
            "norm": WeightSpec((V,), keep=KEEP_FLOAT32, init="one_plus_normal"), "o": WeightSpec((H, V)),
        })
        return specs

    def load_weights(self, tensors):
        t = {n: tensors[n] for n in self.weight_specs()}
        rank = t["w1"].shape[0]
        if t["w2"].shape[1] != rank or rank > ops.CHANNEL_DECAY_MAX_RANK:
            raise ConfigError(f"wkv: the decay's matrices have inner sizes {rank} and {t['w2'].shape[1]}; they must agree and be at most {ops.CHANNEL_DECAY_MAX_RANK}")
        self.mu = self._place(torch.stack([t[f"mu.{s}"].float() for s in MIXES]), KEEP_FLOAT32)
        # products of equal shape run as one launch: all four where keys and values have one size
        if self.k_width == self.v_width:
            self.w_rkvg = self._place(torch.stack([t[s] for s in "rkvg"]), KEEP_COMPUTE)
        else:
            self.w_rk = self._place(torch.stack([t[s] for s in "rk"]), KEEP_COMPUTE)
            self.w_vg = self._place(torch.stack([t[s] for s in "vg"]), KEEP_COMPUTE)
        self.w1 = self._place(t["w1"], KEEP_COMPUTE)
        self.w2t = self._place(t["w2"].float().T.contiguous(), KEEP_FLOAT32)
        self.w0 = self._place(t["w0"], KEEP_FLOAT32)
        self.bonus = self._place(t["u"].reshape(-1), KEEP_FLOAT32)
        self.w_norm = self._place(t["norm"], KEEP_FLOAT32)
        self.w_o = self._place(t["o"], KEEP_COMPUTE)

    def forward(self, h, ctx, cache):
        """``h``: the stream itself (left settled), or ``[T, hidden]`` in the activation dtype."""
        stream = h if isinstance(h, Stream) else Stream(h.float())
        T, dev = stream.residual.shape[0], stream.residual.device
        if stream.gain != 1.0:
            raise ValueError("wkv: a scaled branch output is not folded into the stream by this mixer")
        post_w, post_eps = stream.post if stream.post is not None else (None, 0.0)
        mixes = torch.empty((len(MIXES), T, self.hidden), dtype=self.dtype, device=dev)
        x = ops.settle_shift(stream.residual, stream.pending, post_w, post_eps, cache.state, self.state_floats, ctx.slots, ctx.req_indptr,
                             ctx.token_req, self.mu, mixes)
        stream.residual, stream.pending, stream.post = x, None, None
        K, V = self.k_width, self.v_width
        proj = torch.empty((T, 2 * K + 2 * V), dtype=self.dtype, device=dev)          # r | k | v | gate
        if self.w_rkvg is not None:
            ops.linear_groups(mixes[:4], self.w_rkvg, proj)
        else:
            ops.linear_groups(mixes[:2], self.w_rk, proj[:, : 2 * K])
            ops.linear_groups(mixes[2:4], self.w_vg, proj[:, 2 * K:])
        z = torch.empty((T, self.w1.shape[0]), dtype=torch.float32, device=dev)
        ops.linear(mixes[4], self.w1, None, z)
        decay = torch.empty((T, K), dtype=torch.float32, device=dev)
        ops.channel_decay(z, self.w2t, self.w0, decay)
        o = torch.empty((T, V), dtype=torch.float32, device=dev)
        ops.wkv_scan(proj, K, 2 * K, decay, self.bonus, cache.state, ctx.slots, ctx.req_indptr, o, self.heads, self.dim, self.vdim,
                     max_new_tokens=ctx.max_new_tokens, last_rows=x, tail_off=self.state_floats)
        mixed = torch.empty((T, V), dtype=self.dtype, device=dev)
        ops.gated_head_norm(o, proj[:, 2 * K + V:], self.w_norm, float(self.spec.norm_eps), mixed, self.heads, self.vdim, gate="silu")
        return project_out(mixed, self.w_o, self.dtype)
