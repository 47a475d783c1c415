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


def random_config(seed):
    """a configuration drawn from everything the design allows: widths in whole 64s (so that the fused step takes it) or not, heads, ranks,
    windows and feed-forwards per layer, shared latents in any order"""
    r = np.random.default_rng(1000 + seed)
    pick = lambda *v: int(r.choice(v))  # noqa: E731
    width = pick(64, 128, 256, 320, 448, 576, 1024, 1088) if seed % 3 else pick(40, 100, 152, 260)
    layers, owners = [], []
    for i in range(pick(2, 3, 4)):
        donor = pick(*owners) if owners and r.random() < 0.5 else None
        d = layers[donor][0] if donor is not None else None
        rot = d["rot_dim"] if d else pick(2, 8, 12, 16, 32)
        rank = d["kv_rank"] if d else pick(24, 32, 60, 64, 128, 144, 256, 320)
        base = d["rot"]["base"] if d else float(pick(100, 10000, 1000000))
        m = mixer(pick(1, 2, 3, 4, 6, 8), pick(8, 16, 24, 32, 64, 100), rot, pick(8, 16, 40, 48, 64, 96), rank, pick(3, 17, 31, 32, 33, 64, 65, 128, 500), base=base,
                  kv_from=donor)
        if donor is None:
            owners.append(i)
        layers.append((m, pick(24, 64, 160, 352, 1000, 1408) if r.random() < 0.8 else None))
    return config(width, pick(48, 97, 256, 424, 1000), layers, eps=float(r.choice([1e-6, 1e-5, 1e-3])), cap=float(r.choice([5.0, 15.0, 30.0])))


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
