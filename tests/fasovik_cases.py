"""TEST INFRASTRUCTURE: small configurations of the Fasovik design and checkpoint folders written from random weights."""
import json
import struct

import torch

from oracle import fasovik as O

_NAMES = {torch.bfloat16: "BF16", torch.float32: "F32", torch.int32: "I32"}


def lightning(heads, dim, vdim, decay):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}}


def latent(heads, dim, vdim, rank, scale=None):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "scale": dim ** -0.5 if scale is None else scale}}


def moe(experts, top, ff, identity=None):
    r = {"experts": experts, "top": top}
    if identity is not None:
        r["identity"] = identity
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def config(vocab, width, layers, scale=0.7, mult=0.6, eps=1e-5):
    return {"architecture": "Fasovik", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "residual_mult": mult, "layers": layers}


CONFIGS = {
    # sizes that fit no tile: the general kernels
    "odd": config(131, 76, [dict(lightning(3, 20, 28, [0.5, 0.93, 0.9995]), mlp=moe(5, 3, 44, 2)),
                            dict(latent(3, 18, 26, 34, 0.3), mlp=None),
                            dict(lightning(1, 36, 7, [0.97]), mlp=moe(3, 1, 20))]),
    # sizes the matrix-core kernels take, value dims unlike key dims, a layer used three times
    "tiles": config(320, 384, [dict(latent(6, 64, 96, 160), mlp=moe(6, 2, 128, 1)),
                               dict(lightning(3, 64, 96, [0.61, 0.99, 1.0]), mlp=moe(4, 4, 192)),
                               dict(latent(6, 64, 96, 160), mlp=moe(6, 2, 128, 1), weights_of=0),
                               dict(lightning(2, 128, 64, [0.9, 0.9999]), mlp=None),
                               dict(latent(6, 64, 96, 160), mlp=moe(6, 2, 128, 1), weights_of=2)], mult=1.0),
    # the head and latent sizes of large models
    "large": config(256, 512, [dict(lightning(4, 128, 128, [0.3, 0.95, 0.998, 0.9999]), mlp=moe(8, 3, 256, 2)),
                               dict(latent(8, 128, 128, 512), mlp=moe(9, 4, 384, 3))], scale=1.3, mult=0.4),
    # one of everything
    "ones": config(97, 64, [dict(latent(1, 32, 32, 32, 1.0), mlp=moe(1, 1, 32)),
                            dict(lightning(1, 32, 32, [0.0]), mlp=moe(2, 2, 64, 1))], scale=1.0, mult=1.0, eps=1e-6),
}


def write_folder(path, cfg, tensors):
    """config.json + model.safetensors"""
    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    header, blobs, at = {}, [], 0
    for name, t in tensors.items():
        raw = t.contiguous().flatten().view(torch.uint8).numpy().tobytes()
        header[name] = {"dtype": _NAMES[t.dtype], "shape": list(t.shape), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    head = json.dumps(header).encode()
    (path / "model.safetensors").write_bytes(struct.pack("<Q", len(head)) + head + b"".join(blobs))
    return path


def build(name, dtype, device, tmp_path, seed=0):
    """(config dict, checkpoint tensors, loaded model)"""
    from timeviper_amd.model.llm import load_llm
    cfg = CONFIGS[name]
    tensors = O.random_tensors(cfg, seed)
    return cfg, tensors, load_llm(write_folder(tmp_path / name, cfg, tensors), dtype, device)


def prompt(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def row_errors(got, want):
    """per row: root mean square of the difference, mean taken off, over the spread of the expected logits"""
    d = got.double().cpu() - want.double()
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.double().std()


def run(engine, rid, tokens, cuts):
    """logits of every token of one request, fed in portions of the given sizes (the rest at once)"""
    out, at = [], 0
    for n in list(cuts) + [len(tokens)]:
        part = tokens[at:at + n]
        if part:
            out.append(engine.step([(rid, part, range(len(part)))]).cpu())
            at += len(part)
    return torch.cat(out)
