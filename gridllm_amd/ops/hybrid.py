"""Ops of the layer-list models: HIP kernels for tensors on the GPU, the
PyTorch reference for tensors on the CPU (see hip_hybrid for what each does)."""

from __future__ import annotations

import torch

from gridllm_amd.ops import hip_hybrid, reference_hybrid
from gridllm_amd.ops import reference
from gridllm_amd.ops.reference_hybrid import (  # noqa: F401
    ALL_KEYS, ChunkPortions, Choice, DepthAverage, Keys, StepMeta, Talk)


def _dispatch(name: str):
    hip, ref = getattr(hip_hybrid, name), getattr(reference_hybrid, name)

    def op(t: torch.Tensor, *args, **kw):
        return (hip if t.is_cuda else ref)(t, *args, **kw)

    op.__name__, op.__doc__ = name, hip.__doc__
    return op


embed = _dispatch("embed")
post_norm = _dispatch("post_norm")
sum_norm = _dispatch("sum_norm")
norm_rows = _dispatch("norm_rows")
group_norm = _dispatch("group_norm")
join_norm = _dispatch("join_norm")
poly_norm = _dispatch("poly_norm")
streams_start = _dispatch("streams_start")
streams_join = _dispatch("streams_join")
streams_norm = _dispatch("streams_norm")
proj_f32 = _dispatch("proj_f32")
qknorm_kv = _dispatch("qknorm_kv")
silu_cols = _dispatch("silu_cols")
paged_attn = _dispatch("paged_attn")
latent_rows = _dispatch("latent_rows")
latent_attn = _dispatch("latent_attn")
talk_rows = _dispatch("talk_rows")
talk_attn = _dispatch("talk_attn")
mlstm = _dispatch("mlstm")
gla = _dispatch("gla")
lightning = _dispatch("lightning")
moe = _dispatch("moe")


def glu(gateup: torch.Tensor, p: reference.Glu) -> torch.Tensor:
    """act(gateup[:, :F], gateup[:, F:]) in the input's type."""
    if gateup.is_cuda and gateup.dtype == torch.float32:
        return hip_hybrid.glu_f32(gateup, p)
    from gridllm_amd import ops
    return ops.swiglu(gateup, p)
