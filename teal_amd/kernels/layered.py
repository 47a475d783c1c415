"""Python side of the layered designs' kernels (include/teal_hip.h: teal_layer_*, teal_gated_act, teal_logit_softcap,
teal_latent_*): shape checks, dtype codes and the launch on the current stream.  PyTorch owns every buffer.

Activations and weights fp16, bf16 or true fp32; there is no CPU path."""
from __future__ import annotations

from typing import Optional

import torch

from .. import _lib, runtime

F32 = 2
ACTS = {"silu": 0, "gelu_tanh": 1}
NO_WINDOW = 1 << 30  # a window wider than any sequence: plain causal attention
TILE = 64            # packed key spans of a prompt pass are padded to this many rows


def dtype_code(dt: torch.dtype) -> int:
    return F32 if dt == torch.float32 else runtime.dtype_code(dt)


def _p(t: Optional[torch.Tensor]):
    return None if t is None else t.data_ptr()


def _run(name: str, *args) -> None:
    rc = getattr(_lib.load(), name)(*args, runtime.stream_ptr())
    if rc != 0:
        _lib.check(rc, name)


def _rows(t: torch.Tensor) -> int:
    """row stride of a 2-D tensor whose columns are contiguous"""
    assert t.dim() == 2 and (t.stride(1) == 1 or t.shape[1] == 1), (t.shape, t.stride())
    return t.stride(0)


def resid_norm(x, *, tokens=None, embed=None, y=None, y_bias=None, post_w=None, pre_w=None, eps=1e-6, rows=None, dtype=None):
    """x (fp32 [T, D], in place) = embedding rows | x, + [post norm](y + bias); returns h = RMSNorm(x) * pre_w (rows of `rows`, packed)"""
    assert x.dtype == torch.float32 and x.is_contiguous()
    n = x.shape[0] if rows is None else rows.numel()
    dtype = dtype or (pre_w if pre_w is not None else embed if embed is not None else y).dtype
    h = torch.empty(n, x.shape[1], device=x.device, dtype=dtype) if pre_w is not None else None
    _run("teal_layer_resid_norm", _p(x), n, x.shape[1], _p(tokens), _p(embed), 0 if embed is None else embed.shape[0], _p(y),
         0 if y is None else _rows(y), _p(y_bias), _p(post_w), _p(pre_w), float(eps), _p(h), _p(rows), dtype_code(dtype))
    return h


def gated_act(gu, n_cols: int, up0: int, act: str, bias=None, out=None):
    """act(gate + bias) * (up + bias): gate = gu[:, :n_cols], up = gu[:, up0:up0 + n_cols]; bias laid out like a row of gu"""
    if out is None:
        out = torch.empty(gu.shape[0], n_cols, device=gu.device, dtype=gu.dtype)
    _run("teal_gated_act", _p(gu), _rows(gu), up0, _p(bias), None if bias is None else bias.data_ptr() + up0 * bias.element_size(), _p(out), _rows(out),
         gu.shape[0], n_cols, ACTS[act], dtype_code(gu.dtype))
    return out


def softcap(logits, vocab: int, cap: Optional[float], out=None):
    """fp32 [rows, vocab] = cap * tanh(logits / cap)"""
    if out is None:
        out = torch.empty(logits.shape[0], vocab, device=logits.device, dtype=torch.float32)
    _run("teal_logit_softcap", _p(logits), _rows(logits), _p(out), logits.shape[0], vocab, float(cap or 0.0), dtype_code(logits.dtype))
    return out


def sample_rows(logits, rng, temperature: float, top_k: Optional[int], out=None, pos=None, history=None):
    """one token per row of fp32 logits; rng int64 [rows, 2] {seed, draw counter}; temperature <= 0: the largest logit"""
    assert logits.dtype == torch.float32 and rng.dtype == torch.int64 and rng.is_contiguous() and rng.numel() >= 2 * logits.shape[0]
    if out is None:
        out = torch.empty(logits.shape[0], dtype=torch.int32, device=logits.device)
    _run("teal_sample_rows", _p(logits), _rows(logits), logits.shape[0], logits.shape[1], int(top_k or 0), float(temperature), _p(rng), _p(out), _p(pos), _p(history),
         0 if history is None else history.shape[-1])
    return out


def latent_prompt_rows(proj, kv0, pos, row, inv_freq, norm_w, eps, heads, dim, rot, rank, pool):
    """rotate proj's queries in place; kv0 >= 0: write each token's cache row"""
    assert pos.dtype == torch.int32 and pos.numel() == proj.shape[0]
    _run("teal_latent_prompt_rows", _p(proj), _rows(proj), kv0, proj.shape[0], _p(pos), _p(row), _p(inv_freq), _p(norm_w), float(eps), heads, dim, rot, rank,
         _p(pool), 0 if pool is None else pool.shape[-1], dtype_code(proj.dtype))


def latent_gather(pool, row, rank, rot):
    """(c [n, rank], kr [n, rot]) of the cache rows `row` (negative: zeros)"""
    n = row.numel()
    c = torch.empty(n, rank, device=pool.device, dtype=pool.dtype)
    kr = torch.empty(n, rot, device=pool.device, dtype=pool.dtype)
    _run("teal_latent_gather", _p(pool), pool.shape[-1], _p(row), n, rank, rot, _p(c), _p(kr), dtype_code(pool.dtype))
    return c, kr


def latent_prompt_tile(dim, rot, vdim, n_queries, dtype) -> int:
    return int(_lib.load().teal_latent_prompt_tile(dim, rot, vdim, n_queries, dtype_code(dtype)))


def latent_prompt_attention(q, k, kr, vt, sink, gate, out, seqs, tiles, tile, heads, dim, rot, vdim, window, scale):
    assert k.is_contiguous() and kr.is_contiguous() and vt.is_contiguous() and k.shape[0] == vt.shape[1] == kr.shape[0]
    assert seqs.dtype == tiles.dtype == torch.int32 and seqs.shape[1] == 5 and tiles.shape[1] == 2
    _run("teal_latent_prompt_attention", _p(q), _rows(q), _p(k), _p(kr), _p(vt), k.shape[0], _p(sink), _p(gate), 0 if gate is None else _rows(gate), _p(out),
         _rows(out), _p(seqs), _p(tiles), tiles.shape[0], tile, heads, dim, rot, vdim, int(window), float(scale), dtype_code(q.dtype))
    return out


def latent_qcat(batch, heads, ldq, dtype, device):
    """the absorbed queries' buffer: fp32 rows, or a high and a low 16-bit row"""
    return torch.empty(batch, heads, *(() if dtype == torch.float32 else (2,)), ldq, device=device, dtype=dtype)


def latent_part(batch, heads, splits, rank, device):
    """the splits' partial results: weighted latent (padded to 4), max, sum"""
    return torch.empty(batch * heads * splits * (-(-rank // 4) * 4 + 4), device=device, dtype=torch.float32)


def latent_step_query(proj, kv0, pos, slot, table, page_shift, inv_freq, norm_w, eps, uk, heads, dim, rot, rank, pool, qcat):
    assert uk.is_contiguous() and table.is_contiguous() and pos.dtype == slot.dtype == table.dtype == torch.int32
    _run("teal_latent_step_query", _p(proj), _rows(proj), kv0, proj.shape[0], _p(pos), _p(slot), _p(table), table.shape[1], page_shift, _p(inv_freq), _p(norm_w),
         float(eps), _p(uk), heads, dim, rot, rank, _p(pool), pool.shape[-1], _p(qcat), qcat.shape[-1], dtype_code(proj.dtype))


def latent_step_attention(qcat, pool, pos, slot, table, page_shift, rank, rot, window, scale, splits, part):
    assert part.dtype == torch.float32
    _run("teal_latent_step_attention", _p(qcat), qcat.shape[-1], _p(pool), pool.shape[-1], _p(pos), _p(slot), _p(table), table.shape[1], page_shift, qcat.shape[0],
         qcat.shape[1], rank, rot, int(window), float(scale), splits, _p(part), part.numel() * 4, dtype_code(qcat.dtype))


def latent_step_merge(part, splits, uv, sink, gate, y, batch, heads, rank, vdim):
    assert uv.is_contiguous()
    _run("teal_latent_step_merge", _p(part), splits, _p(uv), _p(sink), _p(gate), 0 if gate is None else _rows(gate), _p(y), _rows(y), batch, heads, rank, vdim,
         dtype_code(y.dtype))
    return y
