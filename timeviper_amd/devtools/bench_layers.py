"""Prefill and decode throughput of the layer-list designs at sizes that resemble a real model's layers, beside the Nemotron
stack at the same width (bench.py --config fasovik | fogorax).

Fasovik: both models get the same number of mixers of each kind (half attention, half recurrence), the same heads x 128 attention,
recurrences of the same inner width and feed-forwards with the same number of active parameters per token.  Fogorax: the other
model is a stack of attention (same heads x 128, all keys visible) and MLP layers whose hidden width makes the parameters per
layer the same.  Random weights.
Per operator: the launches of one step, recorded with their arguments, run back to back between two events (decode: as a
replayed graph), against the HBM roof (8 TB/s) or the dense bf16 MFMA roof (2.5 PFLOP/s) — whichever the algorithmic bytes /
useful FLOPs of the launches make the slower."""
from __future__ import annotations

import json
import time

import torch

HBM, MFMA = 8000.0e9, 2500.0e12

SIZES = {
    "2k": dict(width=2048, heads=16, rank=512, experts=64, identity=8, top=6, ff=1024, layers=8),
    "4k": dict(width=4096, heads=32, rank=512, experts=64, identity=8, top=8, ff=1536, layers=4),
}
FOGORAX_SIZES = {
    "2k": dict(width=2048, heads=16, kv_heads=4, window=1024, keep=64, ff=5632, side=128, layers=8),
    "4k": dict(width=4096, heads=32, kv_heads=8, window=4096, keep=16, ff=9216, side=256, layers=4),
}


def fasovik_config(s):
    import math
    from ..model.llm import FasovikConfig
    ff = {"kind": "moe", "expert": {"ff": s["ff"]}, "router": {"experts": s["experts"], "identity": s["identity"], "top": s["top"]}}
    H = s["heads"]
    decay = [math.exp(-2.0 ** (-8.0 * (h + 1) / H)) for h in range(H)]
    kinds = [{"type": "latent_attention", "mixer": {"heads": H, "dim": 128, "vdim": 128, "kv_rank": s["rank"], "scale": 128 ** -0.5}, "mlp": ff},
             {"type": "lightning", "mixer": {"heads": H, "dim": 128, "vdim": 128, "decay": decay}, "mlp": ff}]
    return FasovikConfig(vocab_size=32768, hidden_size=s["width"], layers=[kinds[i % 2] for i in range(s["layers"])])


def nano_config(s):
    from ..model.llm import NemotronHConfig
    return NemotronHConfig(vocab_size=32768, hidden_size=s["width"], intermediate_size=s["top"] * s["ff"],
                           num_hidden_layers=2 * s["layers"], hybrid_override_pattern="*-M-" * (s["layers"] // 2),
                           num_attention_heads=s["heads"], head_dim=128, num_key_value_heads=s["heads"], ssm_state_size=128,
                           mamba_num_heads=2 * s["heads"], mamba_head_dim=64, mamba_n_groups=8)


def fogorax_config(s, positions):
    """every second layer reads the keys and values of the one in front"""
    from ..model.llm import FogoraxConfig
    layers = []
    for i in range(s["layers"]):
        m = {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
             "mask": {"size": s["window"], "keep_first": s["keep"]}}
        if i % 2:
            m["kv_from"] = i - 1
        layers.append({"type": "attention", "mixer": m, "mlp": {"kind": "dense", "ff": s["ff"]}})
    return FogoraxConfig(vocab_size=32768, hidden_size=s["width"], layers=layers, side_dim=s["side"], max_positions=positions)


def attention_stack_config(s):
    """attention and MLP layers: two matrices of the MLP hold what the gate and the third matrix of a gated feed-forward do"""
    from ..model.llm import NemotronHConfig
    return NemotronHConfig(vocab_size=32768, hidden_size=s["width"], intermediate_size=(3 * s["ff"] + s["heads"] * 128) // 2,
                           num_hidden_layers=2 * s["layers"], hybrid_override_pattern="*-" * s["layers"], num_attention_heads=s["heads"],
                           head_dim=128, num_key_value_heads=s["kv_heads"])


def build(cfg, dev):
    from ..model.llm.llm_factory import llm_class
    with torch.device("meta"):
        llm = llm_class(cfg)(cfg)
    llm = llm.to(torch.bfloat16).to_empty(device=dev)
    g = torch.Generator(device=dev).manual_seed(0)
    with torch.no_grad():
        if hasattr(llm, "init_random"):
            llm.init_random(0)
        else:
            for name, p in llm.named_parameters():
                if name.endswith("A_log"):
                    p.copy_(torch.log(torch.rand(p.shape, device=dev, generator=g) * 15 + 1))
                elif name.endswith("dt_bias"):
                    p.fill_(-4.0)
                elif name.endswith(".D") or "norm" in name.split(".")[-2]:
                    p.fill_(1.0)
                elif name.endswith("bias"):
                    p.zero_()
                else:
                    p.normal_(0.0, 0.02, generator=g)
    return llm.requires_grad_(False).eval()


nb = lambda *ts: sum(t.numel() * t.element_size() for t in ts if t is not None)
size = lambda outs: nb(*[o for o in (outs if isinstance(outs, (tuple, list)) else (outs,)) if torch.is_tensor(o)])


def op_table(K):
    """operator name -> (useful FLOPs, algorithmic bytes) of a call from its arguments and results"""
    def causal(q, k, v, out):
        # (T, H, d) or (B, T, H, d); as many keys as queries
        T, H, d, e = q.shape[-3], q.shape[-2], q.shape[-1], v.shape[-1]
        return T * (T + 1) * H * (d + e) * (q.shape[0] if q.dim() == 4 else 1), nb(q, k, v) + size(out)

    def windowed(res, q, cache, plan, kv_heads, scale, window=K.NO_WINDOW, keep_first=0, **kw):
        # visible pairs; q and o, and the rows of the cache that somebody sees
        T, H, d = q.shape
        e, pairs, seen = cache.shape[2] // kv_heads - d, 0, 0
        for a, n in zip(plan.starts, plan.counts):
            p = torch.arange(a, a + n, dtype=torch.float64)
            lo = (p + 1 - window).clamp(min=0)
            pairs += float((p + 1 - lo + lo.clamp(max=keep_first)).sum())
            seen += a + n - int(lo[0]) + min(keep_first, int(lo[0]))
        return 2 * pairs * H * (d + e), nb(q) + size(res) + seen * cache.shape[2] * 2

    def rows(offsets):
        return int(offsets[-1])

    def used(offsets):
        return int((offsets[1:] > offsets[:-1]).sum())
    t = {
        "attention_sink": lambda out, q, k, v, *a, **kw: causal(q, k, v, out),
        "flash_attn_func": lambda out, q, k, v, *a, **kw: causal(q, k, v, out),
        # one token: the recurrent state in and out; prompts: q, k, v in, o out
        "lightning_attention": lambda out, q, k, v, dec, st, cu, slot, *a, **kw:
            (0, nb(q, k, v) + size(out) + 2 * nb(st[:slot.numel()])),
        "mamba_chunk_scan_combined": lambda out, x, dt, A, B, C, *a, **kw: (0, nb(x, dt, B, C) + nb(out[0])),
        "causal_conv1d_xbc": lambda out, x, *a, **kw: (0, nb(x) + size(out[:3])),
        "rmsnorm_fn": lambda out, x=None, weight=None, bias=None, z=None, **kw: (0, nb(x, z) + size(out)),
        "rms_norm": lambda out, x, w, eps, residual=None, return_sum=False: (0, nb(x, residual) + size(out)),
        "relu2": lambda out, x, **kw: (0, 2 * nb(x)),
        "rms_norm_ex": lambda out, x, w, eps, off=0.0, gate=None, residual=None, y2=None, **kw:
            (0, nb(x, gate, residual) + (size(out) if out is not None and size(out) else nb(x))),
        "moe_combine_norm": lambda out, y, pos, w, res, *a, **kw: (0, int((pos >= 0).sum()) * nb(y[:1]) + nb(res) + size(out)),
        "moe_router": lambda out, x, w, *a, **kw: (2 * x.shape[0] * w.numel(), nb(x, w) + size(out)),
        "moe_plan": lambda out, ids, e: (0, 2 * nb(ids) + size(out)),
        "moe_gemm": lambda out, a, w, offsets, n, **kw:
            (2 * rows(offsets) * w.shape[1] * w.shape[2], used(offsets) * nb(w[0]) + rows(offsets) * (w.shape[1] + w.shape[2]) * 2),
        "linear": lambda out, x, w, *a, **kw: (2 * out.numel() * w.shape[1], nb(x, w) + size(out)),
        # decode
        "gemv_fused": lambda out, x, w, *a, **kw: (0, nb(w)),
        "selective_state_update": lambda out, st, *a, **kw: (0, 2 * nb(st)),
        "flash_attn_decode": lambda out, q, k, v, *a, **kw: (0, nb(k, v)),
        "attention_window": windowed,
        "attention_window_decode": lambda res, *a, **kw: (0, windowed(res, *a, **kw)[1]),
        "norm_shift": lambda out, x, gain, eps, pending=None, *a, **kw: (0, nb(x, pending) + nb(*(t for t in out if t is not x))),
        "residual_add": lambda out, x, u: (0, nb(x, u) + size(out)),
        "gated_mul": lambda res, a, b, *r, **kw: (0, 3 * nb(a)),
        "scatter_rows": lambda out, src, *a: (0, 2 * nb(src)),
        "embed_scaled": lambda out, ids, table, *a, **kw: (0, size(out) + 2 * ids.numel() * table.shape[1] * 2),      # a table row and a position row
        "gemv_pair": lambda out, x, x2, w, *a, **kw: (0, nb(w)),
        "gemv_add": lambda out, x, w, *a: (0, nb(w)),
        "gemv_glu": lambda out, z, u, w, *a, **kw: (0, nb(w)),
        "latent_decode": lambda out, q, uk, uv, lat, keys, slot, *a, **kw: (0, nb(uk, uv) + int(keys.sum()) * lat.shape[2] * 2),
        "gemv_post": lambda out, x, w, *a, **kw: (0, nb(w)),
        # (every choice streams its expert's matrices; the router's weights are the product in front of it)
        "moe_decode": lambda out, z, corr, h, x, up, down, top: (0, len(set(out[1].flatten().tolist()) & set(range(up.shape[0]))) * nb(up[0], down[0])),
    }
    return {k: f for k, f in t.items() if k == "linear" or hasattr(K, k)}


class Recorder:
    """Every call of the table's operators during `with`, with its arguments."""

    def __init__(self):
        from .. import kernels as K
        import torch.nn.functional as F
        self.K, self.F, self.calls, self.depth = K, F, [], 0

    def __enter__(self):
        self.saved = {}
        for name, cost in op_table(self.K).items():
            mod = self.F if name == "linear" else self.K
            self.saved[name] = (mod, getattr(mod, name))
            setattr(mod, name, self._wrap(name, getattr(mod, name), cost))
        return self

    def _wrap(self, name, fn, cost):
        def f(*a, **kw):
            self.depth += 1
            out = fn(*a, **kw)
            self.depth -= 1
            if self.depth == 0:                     # operators inside operators belong to the outer one
                self.calls.append((name, fn, a, kw, cost(out, *a, **kw)))
            return out
        return f

    def __exit__(self, *exc):
        for name, (mod, fn) in self.saved.items():
            setattr(mod, name, fn)

    def rooflines(self, graph: bool, reps: int):
        out = []
        st = torch.cuda.Stream()
        for name in dict.fromkeys(c[0] for c in self.calls):
            mine = [c for c in self.calls if c[0] == name]
            run = lambda: [fn(*a, **kw) for _, fn, a, kw, _ in mine]
            with torch.cuda.stream(st):
                run()
                st.synchronize()
                if graph:
                    g = torch.cuda.CUDAGraph()
                    with torch.cuda.graph(g, stream=st):
                        run()
                    go = g.replay
                else:
                    go = run
                go()
                st.synchronize()
                e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
                e0.record(st)
                for _ in range(reps):
                    go()
                e1.record(st)
                st.synchronize()
            ms = e0.elapsed_time(e1) / reps
            fl, by = sum(c[4][0] for c in mine), sum(c[4][1] for c in mine)
            bound = "mfma" if fl / MFMA > by / HBM else "hbm"
            out.append({"kernel": name, "bound": bound, "launches": len(mine), "ms_per_step": round(ms, 4),
                        "frac": round(max(fl / MFMA, by / HBM) / (ms * 1e-3), 4)})
        return out


def timed(fn, n):
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(n):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t0) / n


@torch.inference_mode()
def measure(llm, T, batch, steps, warm):
    """prefill tokens/s of one prompt of T tokens; decode tokens/s of `batch` sequences of T tokens each; per-operator rooflines"""
    from ..model.llm.decode_graph import GraphedDecodeStep
    dev = llm.device
    ids = torch.randint(0, llm.config.vocab_size, (batch, T), generator=torch.Generator().manual_seed(1)).to(dev)
    pre = lambda c, n=1: llm(input_ids=ids[:n], past_key_values=c, use_cache=True, cache_position=torch.zeros(1, dtype=torch.long))
    for _ in range(warm):
        pre(llm.new_cache(1))
    t = timed(lambda: pre(llm.new_cache(1)), steps)
    with Recorder() as r:
        pre(llm.new_cache(1))
    res = {"prefill_tokens_per_s": round(T / t), "prefill_ms": round(t * 1e3, 3), "prefill_rooflines": r.rooflines(False, 5)}
    res["prefill_accounted"] = round(sum(x["ms_per_step"] for x in res["prefill_rooflines"]) / res["prefill_ms"], 3)
    for b in sorted({1, batch}):
        cache = llm.new_cache(b)
        tok = pre(cache, b).logits[:, -1].argmax(-1).view(b, 1)
        n = 64
        cache.begin_static_decode(n + 16)
        one = torch.ones(1, dtype=torch.long)
        step = GraphedDecodeStep(lambda i: llm(input_ids=i, past_key_values=cache, use_cache=True, cache_position=one).logits, cache, b, dev)
        for _ in range(6):
            tok = step.step(tok)
        assert step.graph is not None, step.capture_error
        t = timed(lambda: step.step(tok), n)
        d = {"tokens_per_s": round(b / t, 1), "ms_per_step": round(t * 1e3, 4)}
        with Recorder() as r:
            llm(input_ids=tok.view(b, 1), past_key_values=cache, use_cache=True, cache_position=one)
        d["rooflines"] = r.rooflines(True, 20)
        res[f"decode_batch_{b}"] = d
        del cache, step
    return res


def main(args):
    from ..build import ensure_built
    ensure_built()
    torch.cuda.set_device(0)
    dev = torch.device("cuda", 0)
    out = {}
    T, batch = args.prompt, args.batch
    steps, warm = max(args.steps, 3), max(args.warmup, 2)
    design = args.config
    for name in args.sizes.split(","):
        s = (SIZES if design == "fasovik" else FOGORAX_SIZES)[name]
        out[name] = {"size": s}
        pair = ((("fasovik", fasovik_config(s)), ("nemotron_hybrid", nano_config(s))) if design == "fasovik" else
                (("fogorax", fogorax_config(s, T + 256)), ("nemotron_attention", attention_stack_config(s))))
        for kind, cfg in pair:
            llm = build(cfg, dev)
            out[name][kind] = measure(llm, T, batch, steps, warm)
            del llm
            torch.cuda.empty_cache()
    first = next(iter(out))
    f = out[first][design]
    print(json.dumps({
        "metric": f"prefill tokens/s, {design.capitalize()} layers at width {out[first]['size']['width']}, one prompt", "value": f["prefill_tokens_per_s"],
        "unit": "tokens/s", "n_gpus": 1, "steps": steps, "warmup": warm, "ms_per_step": f["prefill_ms"], "higher_is_better": True,
        "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
        "config": {"prompt_tokens": T, "decode_batches": sorted({1, batch}), "weights": "random init, seed 0"}, "sizes": out}), flush=True)
