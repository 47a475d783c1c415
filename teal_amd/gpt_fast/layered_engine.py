"""Fused HIP decode step of the layered designs at batch 1, 16-bit: engine.DecodeEngine's counterpart for layered.LayeredTransformer.

A layer with latent attention and a gated feed-forward is seven launches; everything between two matrix products is folded into
the consumer's producer or epilogue, over an fp32 residual:

  1. proj    [x += norm1b-of-last(down slabs + bias); h = RMSNorm(x) * norm1] -> mask(tau_q|g|kv) -> GEMV -> q | gate | latent
  2. query   W_uk^T q per head, rotation; the token's cache row (norm of the latent, rotated key part)
  3. attend  split over the cached rows of the window                                                   -> fp32 partials
  4. merge   partials + sink -> W_uv -> * sigmoid(gate)                                                 -> y
  5. wo      mask(tau_o) -> GEMV                                                                        -> fp32 slabs
  6. gate|up [x += norm1b(wo slabs); h = RMSNorm(x) * norm2] -> mask(tau_gate|up) -> GEMV, + bias, gelu -> gelu(gate) | up
  7. down    [gelu(gate) * up] -> mask(tau_down) -> GEMV                                                -> fp32 slabs
  head       [x += norm2b(down slabs + bias); h = RMSNorm(x) * norm] -> GEMV -> fp32 logits, soft cap

Launches 1, 5, 6, 7 and the head are the framework's masked GEMV (teal_fused_gemv) over the same column-major weight images, so
activation sparsity applies to this design as to the others: `thresholds[i]` = {"q", "g", "kv", "o", "gate", "up", "down": tau}.
"""
from __future__ import annotations

import ctypes
from typing import Dict, List, Optional

import torch

from .. import _lib, runtime
from ..kernels import layered as K
from .engine import (MAX_SLABS, TEAL_IN_PLAIN, TEAL_IN_RESID32_NORM, TEAL_IN_SILU_MUL, TEAL_OUT_ROUNDED, TEAL_OUT_SLAB_SUM, TEAL_OUT_SLABS, DecodeLoop, GemvIn,
                     _out)
from .layered import GatedMLP, LatentAttention, LayeredTransformer, StepBatch, pad_to

SITES = ("q", "g", "kv", "o", "gate", "up", "down")
KEEP_ALL = float("-inf")
ACT_SEG0 = {"gelu_tanh": 2}


class LayeredEngine(DecodeLoop):
    reduce = None
    tp_world = 1

    @staticmethod
    def supports(model: LayeredTransformer, need_caches: bool = True) -> Optional[str]:
        """None if the fused step can run `model`, else the reason (the caller keeps the unfused step)"""
        w, cfg = model.tok_embeddings.weight, model.config
        if w.dtype not in (torch.float16, torch.bfloat16):
            return f"weights are {w.dtype} (the fused step is built for fp16 / bf16)"
        if not w.is_cuda:
            return "model is not on a HIP device"
        if cfg.dim % 64 or cfg.dim > 8192:
            return f"width {cfg.dim} (need a multiple of 64, <= 8192)"
        if not cfg.design.post_norms:
            return "sublayer outputs without a norm of their own"
        for b in model.layers:
            if not isinstance(b.mix, LatentAttention) or not (b.mlp is None or isinstance(b.mlp, GatedMLP)):
                return f"no fused form of {type(b.mix).__name__} / {type(b.mlp).__name__}"
            if b.mlp is not None and (b.mlp.a.act not in ACT_SEG0 or b.mlp.fp > 65536):
                return f"feed-forward {b.mlp.a.act}, {b.mlp.fp} wide"
            if b.mix.nv > 65536:
                return f"{b.mix.nv} attention outputs"
        if need_caches and model.cache is None:
            return "caches are not set up (model.setup_caches)"
        return None

    def __init__(self, model: LayeredTransformer, thresholds: Optional[List[Dict[str, float]]] = None, cache=None, max_seq: Optional[int] = None, **_):
        why = LayeredEngine.supports(model, need_caches=cache is None)
        if why is not None:
            raise ValueError(f"LayeredEngine cannot run this model: {why}")
        self.L = _lib.load()
        runtime.init()
        self.model, self.cfg = model, model.config
        self.cache = model.cache if cache is None else cache
        self.max_seq = max_seq or model.max_seq_length
        w = model.tok_embeddings.weight
        dev, dt, dim = w.device, w.dtype, self.cfg.dim
        self.dim, self.dtype, self.code = dim, torch.float32, runtime.dtype_code(dt)  # (dtype: of the logits)
        z = lambda *shape, dtype=dt: torch.zeros(*shape, device=dev, dtype=dtype)  # noqa: E731
        mixes, mlps = [b.mix for b in model.layers], [b.mlp for b in model.layers if b.mlp is not None]
        self.resid = [z(dim, dtype=torch.float32), z(dim, dtype=torch.float32)]
        self.proj = z(1, max(m.proj.out_features for m in mixes))
        self.ys = {n: z(1, n) for n in {m.wo.in_features for m in mixes}}  # (columns past a mixer's outputs stay zero)
        self.gu = z(max([2 * m.fp for m in mlps], default=8))
        self.slabs = [z(MAX_SLABS, dim, dtype=torch.float32), z(MAX_SLABS, dim, dtype=torch.float32)]
        self.qcat = {}
        for m in mixes:
            key = (m.a.heads, self.cache.pools[m.owner].shape[-1])
            self.qcat[key] = K.latent_qcat(1, *key, dt, dev)
        self.part = max((K.latent_part(1, m.a.heads, m.MAX_SPLITS, m.a.kv_rank, dev) for m in mixes), key=torch.numel)
        self.vocab_pad = model.output.weight.shape[0]
        self.logits_pad = z(self.vocab_pad, dtype=torch.float32)
        self.logits = self.logits_pad[: self.cfg.vocab_size].view(1, 1, -1)
        self.ws = runtime.new_workspace(max([dim] + [m.fp for m in mlps]), max([self.vocab_pad, self.proj.numel(), self.gu.numel()]))
        self.slot = torch.zeros(1, dtype=torch.int32, device=dev)
        self.max_pos = self.max_seq - 1  # (chooses how far the attention is split)
        self.eps = float(self.cfg.norm_eps)
        self._n = ctypes.c_int(0)
        self._init_loop(dev)
        self._build(thresholds or [dict.fromkeys(SITES, KEEP_ALL) for _ in mixes])

    # ---- static launch descriptors ---------------------------------------------------------------------------------
    def _build(self, ths: List[Dict[str, float]]) -> None:
        m, A, B = self.model, *self.resid
        zero = torch.zeros_like(m.norm)
        self.thresholds, self._keep, self.launches = ths, [], []
        prev = None       # (post-norm weight, bias) of the sublayer whose slabs the next producer folds into the residual
        src, dst = A, B   # the residual ping-pongs between two buffers
        sub = 0

        def producer(pre):
            nonlocal src, dst
            post, bias = prev if prev is not None else (zero, zero)
            vec3 = torch.stack([pre, post, zero if bias is None else bias]).contiguous()
            self._keep.append(vec3)
            gin = GemvIn(mode=TEAL_IN_RESID32_NORM, slabs=None if prev is None else self.slabs[(sub + 1) & 1].data_ptr(), nslabs=0, slabs_interleaved=1,
                         norm_weight=vec3.data_ptr(), eps=self.eps, resid_in=(m.tok_embeddings.weight if prev is None else src).data_ptr(), resid_out=dst.data_ptr())
            src, dst = dst, src
            return gin

        def seg(lin, col0, ncols, tau, y):
            w = lin.weight
            return (w.data_ptr(), w.stride(1), col0, ncols, tau, None if y is None else y.data_ptr() + y.element_size() * col0)

        for layer, th in zip(m.layers, ths):
            mix = layer.mix
            cuts = [(0, mix.g0, "q"), (mix.g0, mix.kv0, "g"), (mix.kv0, mix.proj.out_features, "kv")]
            gin = producer(layer.norm1)
            gout = _out([seg(mix.proj, lo, hi - lo, th[n], self.proj) for lo, hi, n in cuts if hi > lo], TEAL_OUT_ROUNDED)
            y = self.ys[mix.wo.in_features]
            win = GemvIn(mode=TEAL_IN_PLAIN, x=y.data_ptr())
            wout = _out([seg(mix.wo, 0, self.dim, th["o"], None)], TEAL_OUT_SLABS, self.slabs[sub & 1])
            prev, sub = (layer.norm1b, None), sub + 1
            ff = None
            if layer.mlp is not None:
                mlp = layer.mlp
                fin = producer(layer.norm2)
                fout = _out([seg(mlp.gate_up, 0, mlp.fp, th["gate"], self.gu), seg(mlp.gate_up, mlp.fp, mlp.fp, th["up"], self.gu)], TEAL_OUT_ROUNDED)
                fout.act_seg0 = ACT_SEG0[mlp.a.act]
                fout.bias = None if mlp.gate_up_bias is None else mlp.gate_up_bias.data_ptr()
                din = GemvIn(mode=TEAL_IN_SILU_MUL, x=self.gu.data_ptr(), gate_activated=1)
                dout = _out([seg(mlp.down, 0, self.dim, th["down"], None)], TEAL_OUT_SLABS, self.slabs[sub & 1])
                ff = (fin, fout, din, dout, mlp.fp)
                prev, sub = (layer.norm2b, mlp.down_bias), sub + 1
            self.launches.append((mix, gin, gout, y, win, wout, ff))
        hin = producer(m.norm)
        hin.resid_out = None
        hout = _out([seg(m.output, 0, self.vocab_pad, KEEP_ALL, None)], TEAL_OUT_SLAB_SUM)
        hout.slabs, hout.slabs_bytes = self.logits_pad.data_ptr(), self.logits_pad.numel() * 4
        hout.softcap = self.cfg.logit_softcap or 0.0
        self.head = (hin, hout)

    def _gemv(self, gin, gout, Z: int) -> int:
        rc = self.L.teal_fused_gemv(ctypes.byref(gin), ctypes.byref(gout), Z, self.code, self.ws.data_ptr(), self.ws.numel() * 4, ctypes.byref(self._n), self._stream)
        if rc != 0:
            _lib.check(rc, "teal_fused_gemv")
        return self._n.value

    STAGES = ("proj", "attend", "wo", "gate_up", "down", "head")

    def __call__(self, idx: torch.Tensor, input_pos: torch.Tensor, only=STAGES) -> torch.Tensor:
        """idx: int32 [1, 1] token id, input_pos: int32 [1] position -> logits [1, 1, vocab] (fp32; the next call overwrites them).
        `only` (measurements: stage_times): launch just these stages, on whatever the buffers hold from the last full step."""
        assert idx.dtype == torch.int32 and input_pos.dtype == torch.int32 and idx.numel() == 1
        self._stream = runtime.stream_ptr()
        b = StepBatch(self.cache, idx, input_pos, self.slot, self.max_pos)
        slabs = 0
        for i, (mix, gin, gout, y, win, wout, ff) in enumerate(self.launches):
            if i == 0:
                gin.row_index = idx.data_ptr()
            if "proj" in only:
                gin.nslabs = slabs
                self._gemv(gin, gout, self.dim)
            if "attend" in only:
                mix.attend(self.proj[:, : mix.proj.out_features], b, y, (self.qcat[(mix.a.heads, self.cache.pools[mix.owner].shape[-1])], self.part))
            if "wo" in only:
                slabs = self._gemv(win, wout, mix.wo.in_features)
            if ff is not None:
                fin, fout, din, dout, Z = ff
                if "gate_up" in only:
                    fin.nslabs = slabs
                    self._gemv(fin, fout, self.dim)
                if "down" in only:
                    slabs = self._gemv(din, dout, Z)
        if "head" in only:
            hin, hout = self.head
            hin.nslabs = slabs
            self._gemv(hin, hout, self.dim)
        return self.logits

    @torch.no_grad()
    def stage_times(self, reps: int = 20) -> Dict[str, Dict[str, float]]:
        """Microseconds per launch group and layer — a hipGraph of that one stage over every layer, its launch boundaries included — and
        the bytes a dense step has to move for it.  Run after a full step: a stage works on what the buffers hold."""
        m, out, el = self.model, {}, 2
        pos = int(self.pos_buf.item())
        mean = lambda f: sum(f(b) for b in m.layers) / len(m.layers)  # noqa: E731

        def attention_bytes(b):
            a = b.mix.a
            keys = min(pos + 1, b.mix.window)
            return el * (b.mix.uk.numel() + b.mix.uv.numel() + keys * (a.kv_rank + a.rot_dim) + b.mix.proj.out_features + b.mix.nv)

        size = {"proj": mean(lambda b: el * b.mix.proj.weight.numel()), "attend": mean(attention_bytes), "wo": mean(lambda b: el * b.mix.wo.weight.numel()),
                "gate_up": mean(lambda b: el * b.mlp.gate_up.weight.numel() if b.mlp is not None else 0),
                "down": mean(lambda b: el * b.mlp.down.weight.numel() if b.mlp is not None else 0), "head": el * m.output.weight.numel()}
        for stage in self.STAGES:
            s = torch.cuda.Stream()
            s.wait_stream(torch.cuda.current_stream())
            with torch.cuda.stream(s):
                self(self.tok_buf, self.pos_buf, only=(stage,))
            torch.cuda.current_stream().wait_stream(s)
            torch.cuda.synchronize()
            g = torch.cuda.CUDAGraph()
            with runtime.graph_capture(g):
                self(self.tok_buf, self.pos_buf, only=(stage,))
            ts = []
            for r in range(reps + 3):
                e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
                e0.record()
                g.replay()
                e1.record()
                e1.synchronize()
                if r >= 3:
                    ts.append(e0.elapsed_time(e1) * 1e3 / (1 if stage == "head" else len(m.layers)))
            out[stage] = {"us": sorted(ts)[len(ts) // 2], "bytes": size[stage]}
        return out

    def sample_fused(self, logits: torch.Tensor, temperature: float = 1.0, top_k: Optional[int] = None, feed: bool = False) -> torch.Tensor:
        tok = self.tok_buf if feed else self.token
        K.sample_rows(logits.view(1, -1), self.rng_state, max(float(temperature), 0.0), top_k, tok, self.pos_buf if feed else None, self.history if feed else None)
        return tok


@torch.no_grad()
def calibrate_thresholds(model: LayeredTransformer, sparsity: float, n_tokens: int = 64, seed: int = 4321) -> List[Dict[str, float]]:
    """Per layer and projection the `sparsity` quantile of |activation| over a short dense prompt of random tokens (synthetic
    calibration, as generate.calibrate_thresholds does for the Llama stack)."""
    if sparsity <= 0:
        return [dict.fromkeys(SITES, KEEP_ALL) for _ in model.layers]
    from .serving import BatchEngine
    taus, hooks = [dict.fromkeys(SITES, KEEP_ALL) for _ in model.layers], []

    def watch(lin, n, i, names):
        def pre(_m, args):
            a = args[0][:, :n].detach().float().abs().flatten()  # (columns past n are padding)
            t = float(torch.quantile(a[:: max(1, a.numel() // 200000)], sparsity))
            taus[i].update(dict.fromkeys(names, t))
        hooks.append(lin.register_forward_pre_hook(pre))

    for i, b in enumerate(model.layers):
        watch(b.mix.proj, model.config.dim, i, ("q", "g", "kv"))
        watch(b.mix.wo, b.mix.nv, i, ("o",))
        if b.mlp is not None:
            watch(b.mlp.gate_up, model.config.dim, i, ("gate", "up"))
            watch(b.mlp.down, b.mlp.a.ff, i, ("down",))
    toks = torch.randint(0, model.config.vocab_size, (n_tokens,), generator=torch.Generator().manual_seed(seed)).tolist()
    BatchEngine(model, n_tokens).step([(0, toks, [n_tokens - 1])])
    for h in hooks:
        h.remove()
    return taus
