"""TEST INFRASTRUCTURE: small configurations of the Fogorax design and checkpoint folders written from random weights."""
from fasovik_cases import prompt, row_errors, run, write_folder  # noqa: F401
from oracle import fogorax as O


def layer(heads, kv_heads, dim, vdim, size, keep=0, ff=None, kv_from=None, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale,
         "mask": {"size": size, "keep_first": keep}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(vocab, width, layers, side, positions=700, eps=1e-5):
    return {"architecture": "Fogorax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "token_side": {"dim": side},
            "max_positions": positions, "layers": layers}


CONFIGS = {
    # sizes that fit no tile: the general kernels; a shared cache read through another window, a layer without feed-forward
    "odd": config(131, 76, [layer(6, 3, 18, 22, 9, 3, 44, scale=0.3), layer(6, 3, 18, 22, 14, 0, None, kv_from=0),
                            layer(1, 1, 10, 7, 5, 1, 20), layer(6, 3, 18, 22, 4, 6, 30, kv_from=0)], 10),
    # sizes the matrix-core kernels take, value dims unlike key dims, windows around the tiles' edges
    "tiles": config(320, 384, [layer(8, 2, 64, 96, 65, 5, 256), layer(8, 2, 64, 96, 33, 0, 320, kv_from=0), layer(4, 4, 96, 40, 97, 100, 128),
                               layer(8, 2, 64, 96, 200, 1, None, kv_from=0), layer(4, 4, 96, 40, 20, 2, 200, kv_from=2)], 24),
    # head sizes of large models; one key / value head for many query heads
    "large": config(256, 512, [layer(8, 4, 128, 128, 130, 70, 640), layer(12, 1, 128, 64, 40, 3, 512, scale=0.12),
                               layer(8, 4, 128, 128, 300, 0, 384, kv_from=0)], 64),
    # one of everything; a window of one token, nothing kept
    "ones": config(97, 64, [layer(1, 1, 32, 32, 1, 0, 32, scale=1.0), layer(1, 1, 8, 8, 2, 1, None, scale=1.0)], 8, positions=40, eps=1e-6),
    # rows the matrix-vector kernels take around heads the attention kernels do not
    "mixed": config(75, 64, [layer(2, 2, 20, 12, 11, 2, 40), layer(4, 2, 12, 18, 30, 0, 24), layer(2, 2, 20, 12, 300, 0, 16, kv_from=0)], 16),
    # heads wider than the prompt kernel's tiles; everything visible
    "wide": config(80, 128, [layer(2, 1, 192, 256, 500, 0, 72), layer(3, 3, 256, 136, 17, 4, None)], 16),
}


def build(name, dtype, device, tmp_path, seed=0):
    """(config dict, checkpoint tensors, loaded model)"""
    from timeviper_amd.model.llm import load_llm
    cfg = CONFIGS[name]
    tensors = O.random_tensors(cfg, seed)
    return cfg, tensors, load_llm(write_folder(tmp_path / name, cfg, tensors), dtype, device)
