"""Small random models of the layered designs for the tests: configurations with sizes of their own, weights that make single keys
stand out, and the checkpoint folder the framework loads them from."""
import json
import math

import numpy as np
import torch


def mixer(heads, dim, rot, vdim, rank, window, base=10000.0, scale=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "mask": {"size": window}, "rot": {"base": base, "dims": rot},
         "scale": (dim + rot) ** -0.5 if scale is None else scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def config(width, vocab, layers, eps=1e-5, cap=20.0):
    """layers: [(mixer, ff or None)]"""
    return {"architecture": "Bolizen", "width": width, "vocab": vocab, "norm": {"eps": eps}, "logit_softcap": cap,
            "layers": [{"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None} for m, ff in layers]}


CONFIGS = {
    # every layer different: sizes that are no multiples of 8, shared latents out of order, layers without a feed-forward
    "ragged": config(72, 101, [(mixer(3, 20, 6, 28, 36, 33), 52), (mixer(2, 11, 6, 9, 36, 7, kv_from=0), None), (mixer(1, 16, 4, 12, 20, 70, base=500.0, scale=0.4), 30),
                               (mixer(5, 8, 6, 20, 36, 64, kv_from=0), 90), (mixer(2, 24, 4, 33, 20, 1, base=500.0, kv_from=2), 41)], eps=3e-3, cap=7.0),
    # whole tiles throughout; one shared cache, windows of a page, a page and one, less than a tile
    "even": config(128, 256, [(mixer(4, 32, 16, 32, 64, 64), 192), (mixer(2, 48, 16, 64, 64, 65, kv_from=0), 128), (mixer(4, 16, 32, 16, 96, 20, base=2000.0), 256)], cap=12.0),
    # more than sixteen heads, a latent that is no multiple of 16 and one larger than 256
    "heads": config(192, 320, [(mixer(20, 24, 8, 16, 200, 40), 128), (mixer(17, 16, 8, 24, 200, 100, kv_from=0), None), (mixer(3, 64, 32, 80, 320, 96), 320)]),
    # head sizes and latents at the far end of the matrix-core tiles, and (second and third layer) beyond them
    "large": config(256, 200, [(mixer(2, 160, 96, 144, 512, 50), 96), (mixer(1, 200, 64, 264, 520, 45), 64),
                               (mixer(2, 16, 8, 16, 1060, 30), None)]),
}


def random_tensors(cfg, seed=0, peak=3.0):
    """bf16 weights: matrices N(0, 1 / inputs), the query projections `peak` times that (one score stands out per query), norm weights
    around 1, biases and sinks of order 1"""
    from teal_amd.gpt_fast.layered import LayeredArgs, LayeredTransformer
    with torch.device("meta"):
        shapes = LayeredTransformer(LayeredArgs.from_dict(cfg)).tensor_shapes()
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes.items():
        r = torch.randn(shape, generator=g)
        if name.endswith("norm") or ".norm" in name:
            t = 1.0 + 0.3 * r
        elif name.endswith(".sink"):
            t = 1.0 + r
        elif len(shape) == 1:
            t = 0.5 * r
        elif name == "embed":
            t = 2.0 * r
        else:
            t = r / math.sqrt(shape[1]) * (peak if name.endswith(".q") else 1.0)
        out[name] = t.to(torch.bfloat16)
    return out


def save_checkpoint(folder, cfg, tensors):
    from safetensors.torch import save_file
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in tensors.items()}, str(folder / "model.safetensors"))
    return folder


def random_tokens(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


def error(got, want):
    """per position: rms of the difference over the vocabulary, relative to the rms of the expected logits"""
    got, want = got.detach().double().cpu(), want.double()
    return ((got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt())
