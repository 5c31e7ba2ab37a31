#!/usr/bin/env python3
"""Benchmark of the W4A32 quantized-Linear hot path on one MI355X.

A "step" is one decode token's worth of W4A32 Linears at M=1 on Qwen2-1.5B shapes: 28 layers
x {q, k, v, o, gate, up, down} + lm_head, every layer with its own weights (868 MB of
nibbles+scales per step, more than the 256 MB Infinity Cache, so weights come from HBM as
they do in real decoding). Each Linear is the whole op (per-row int8 quantisation of the
activations + the product); Linears that take the same input (q,k,v and gate,up) are issued
as one grouped call, as a decoder would. `extra.one_launch_per_linear` is the same pass with
one call per Linear.

Prints ONE JSON line. `value` = algorithmic bytes of the step / time per step (GB/s), inputs
resident in HBM. `roofline` = the decode kernel (gemv_fused_kernel: row quantisation + product
in one launch, the only kernel in the step) over the same launches, timed with HIP events on
the launch stream, against 8 TB/s. `extra` carries per-shape decode figures, the M=512 and
M=2048 prefill TFLOP/s (whole op and product kernel alone) and the prefill kernel's MFMA
roofline. `cpu_baseline` = the scalar CPU restatement of the reference path on this host, on a
bounded sample.
"""
import argparse
import importlib
import json
import numpy as np
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)

HBM_PEAK_GBS = 8000.0
# HBM bytes per launch of the decode pass, measured with hardware counters (not re-measured by a
# bench run: the counters need the profiler); algorithmic bytes per launch are 7,732,011.
PASS_TRAFFIC_BYTES_PER_LAUNCH = 8003128
LAYERS = 28
# name, K, N, bias, count per layer
LAYER_LINEARS = [
    ("q_proj", 1536, 1536, True),
    ("k_proj", 1536, 256, True),
    ("v_proj", 1536, 256, True),
    ("o_proj", 1536, 1536, False),
    ("gate_proj", 1536, 8960, False),
    ("up_proj", 1536, 8960, False),
    ("down_proj", 8960, 1536, False),
]
LM_HEAD = ("lm_head", 1536, 151936, False)


def algorithmic_bytes(M, K, N, bias):
    """nibbles + bf16 block scales (+ bias) + activations in + outputs out."""
    return N * K // 2 + N * (K // 32) * 2 + (N * 4 if bias else 0) + M * K * 4 + M * N * 4


def parse():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=50)
    ap.add_argument("--warmup", type=int, default=5)
    ap.add_argument("--no-cpu", action="store_true", help="skip the CPU baseline leg")
    ap.add_argument("--no-gemm", action="store_true", help="skip the prefill (M=512) leg")
    ap.add_argument("--eager", action="store_true", help="launch from Python instead of a HIP graph")
    ap.add_argument("--roofline-only", action="store_true",
                    help="only the decode passes (the run profiled under rocprofv3 --kernel-trace)")
    ap.add_argument("--no-decoder", action="store_true", help="skip the whole-decoder tokens/s leg")
    ap.add_argument("--pass", dest="which_pass", choices=("auto", "split", "unsplit"), default="auto",
                    help="decode pass to time: down_proj split over K, unsplit, or both and the faster one "
                         "(auto); a profiled run names one so that its trace holds a single pass shape")
    ap.add_argument("--traffic-probe", action="store_true",
                    help="a 256 MiB copy, then the decode kernel on gate_proj and lm_head and the "
                         "prefill kernel on gate_proj and down_proj (the run profiled under rocprofv3 --pmc)")
    ap.add_argument("--layered", metavar="SIZES", nargs="?", const="small,mid,large", default=None,
                    help="instead of the default workload: prefill and decode of the layered decoder (pooled-window "
                         "attention / gated delta rule / retention, bf16) beside the W4A32 decoder of equal size; "
                         "SIZES: comma-separated names of LAYERED_SIZES")
    ap.add_argument("--lesarax", metavar="SIZES", nargs="?", const="small,mid,large", default=None,
                    help="instead of the default workload: prefill and decode of a decoder with latent and rotary attention, "
                         "experts and looped layers (bf16) beside the layered decoder of equal size; SIZES as for --layered")
    ap.add_argument("--layered-only", choices=("both", "layered", "w4a32", "lesarax"), default="both",
                    help="with --layered or --lesarax: run one of the two models (for a profile of it alone)")
    return ap.parse_args()


# name -> hidden, heads, kv heads, feed-forward, layers, vocab (heads of 128)
LAYERED_SIZES = {
    "small": (1024, 8, 2, 4096, 24, 65536),
    "mid": (1536, 12, 2, 8960, 28, 151936),
    "large": (3584, 28, 4, 18944, 28, 152064),
}


def layered_model(torch, size, gen):
    """config.json's dictionary and random bf16 weights of a layered decoder: attention, delta and retention layers
    in turn, every second attention layer reading the keys and values of the one before it."""
    W, H, G, F, L, V = size
    layers, last_kv = [], None
    for i in range(L):
        kind = ("attention", "delta", "retention")[i % 3]
        m = {"heads": H, "dim": 128, "vdim": 128}
        if kind == "attention":
            m.update(kv_heads=G, conv=4, scale=128 ** -0.5, mask={"size": 1024, "pool": 16})
            if last_kv is None:
                last_kv = i
            else:
                m["kv_from"], last_kv = last_kv, None
        elif kind == "delta":
            m.update(kv_heads=H // 2, conv=4)
        else:
            m.update(decay=[1 - 2.0 ** -(5 + 5 * h / H) for h in range(H)], rot={"dims": 128, "base": 1e6})
        layers.append({"type": kind, "mixer": m, "mlp": {"kind": "dense", "ff": F}})
    cfg = {"architecture": "Suripel", "width": W, "vocab": V, "canon": {"taps": 4}, "norm": {"eps": 1e-5},
           "layers": layers}

    def rnd(*shape, std=0.02):
        return (torch.randn(shape, generator=gen, device="cuda") * std).to(torch.bfloat16)
    one = lambda n: torch.ones(n, device="cuda")
    w = {"embed": rnd(V, W, std=1.0), "head": rnd(V, W), "final.norm": one(W)}
    for i, layer in enumerate(layers):
        m, p, kind = layer["mixer"], f"l{i}.", layer["type"]
        kv = m.get("kv_heads", H)
        nq = (kv if kind == "delta" else H) * 128
        parts = {"q": nq}
        if m.get("kv_from") is None:
            parts.update(k=kv * 128, v=(kv if kind == "attention" else H) * 128)
        for n, rows in parts.items():
            w[p + "mix." + n] = rnd(rows, W)
            if "conv" in m:
                w[p + f"mix.{n}.conv"] = rnd(rows, m["conv"], std=0.4)
        if kind != "attention":
            w[p + "mix.g"] = rnd(H * 128, W)
        if kind == "delta":
            w[p + "mix.a"], w[p + "mix.b"] = rnd(H, W), rnd(H, W)
            w[p + "mix.A_log"], w[p + "mix.dt_bias"], w[p + "mix.norm"] = rnd(H), rnd(H) - 3, one(128)
        w[p + "mix.o"] = rnd(W, H * 128)
        w[p + "mlp.up"], w[p + "mlp.down"] = rnd(F, W), rnd(W, F)
        w[p + "mlp.act"] = torch.tensor([0.3, 0.3, 0.3, 0.0], device="cuda")
        for n in ("norm1", "norm2"):
            w[p + n] = one(W)
        for n in ("canon1", "canon2"):
            w[p + n] = rnd(W, 4, std=0.3)
    matrix = sum(t.numel() for t in w.values() if t.ndim == 2 and t.shape[1] > 8) - V * W  # the embedding is gathered
    return cfg, w, matrix


def lesarax_model(torch, size, gen):
    """As layered_model for Lesarax: as many layer runs (the middle half of them two passes through a quarter of the layers),
    three latent layers to one of rotary attention, 16 experts of a quarter of the feed-forward's width of which 4 run."""
    W, H, G, F, L, V = size
    q_rank, kv_rank, rot = W // 2, 512 if W > 2000 else 256, 64
    start = quarter = L // 4
    n = L - quarter
    mlp = {"kind": "moe", "expert": {"ff": F // 4, "limit": 7.0}, "router": {"experts": 16, "top": 4}}
    layers = []
    for i in range(n):
        if i % 4 == 2:
            m = {"heads": H, "kv_heads": G, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "rot": {"dims": rot, "base": 1e6}}
            layers.append({"type": "attention", "mixer": m, "mlp": mlp})
        else:
            m = {"heads": H, "dim": 128, "rot_dim": rot, "vdim": 128, "q_rank": q_rank, "kv_rank": kv_rank,
                 "scale": (128 + rot) ** -0.5, "mask": {"size": 1024}, "rot": {"dims": rot, "base": 1e6}}
            layers.append({"type": "latent_attention", "mixer": m, "mlp": mlp})
    cfg = {"architecture": "Lesarax", "width": W, "vocab": V, "norm": {"eps": 1e-5}, "residual_mult": 0.5,
           "loop": {"start": start, "stop": start + quarter, "times": 2}, "layers": layers}

    def rnd(*shape, std=0.02):
        return (torch.randn(shape, generator=gen, device="cuda") * std).to(torch.bfloat16)
    one = lambda n: torch.ones(n, device="cuda")
    w = {"embed": rnd(V, W, std=1.0), "final.norm": one(W), "loop.in": rnd(W, 2 * W)}
    body = 0                                    # elements of the matrices one token meets in the layers' runs
    for i, layer in enumerate(layers):
        m, p, q = layer["mixer"], f"l{i}.", f"l{i}.mix."
        if layer["type"] == "attention":
            shapes = {"q": (H * 128, W), "k": (G * 128, W)}
        else:
            shapes = {"dq": (q_rank, W), "uq": (H * (128 + rot), q_rank), "dkv": (kv_rank + rot, W),
                      "uk": (H * 128, kv_rank), "uv": (H * 128, kv_rank), "g": (H, W)}
            w[q + "dq.norm"], w[q + "dkv.norm"] = one(q_rank), one(kv_rank)
        shapes["o"] = (W, H * 128)
        for name, shape in shapes.items():
            w[q + name] = rnd(*shape)
        w[q + "sink"] = rnd(H, std=1.0)
        w[p + "norm1"], w[p + "norm2"], w[p + "mlp.router"] = one(W), one(W), rnd(16, W)
        for e in range(16):
            w[f"{p}mlp.e{e}.gate"], w[f"{p}mlp.e{e}.up"] = rnd(F // 4, W), rnd(F // 4, W)
            w[f"{p}mlp.e{e}.down"] = rnd(W, F // 4)
        runs = 2 if start <= i < start + quarter else 1
        body += runs * (sum(a * b for a, b in shapes.values()) + 16 * W + 3 * F * W)
    return cfg, w, body + 2 * 2 * W * W + V * W


def layered_bench(args, torch, pkg):
    gen = torch.Generator(device="cuda")
    gen.manual_seed(7)
    stream = torch.cuda.Stream()
    e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    max_seq, n_new, prompts = 4096, 128, (512, 2048)

    def measure(prefill, step, prepare):
        """ms per prefill of each length, ms per greedy step behind a 2048-token prompt (graph replay)."""
        out = {}
        torch.cuda.synchronize()                # weights and workspace are made on the default stream
        with torch.cuda.stream(stream):
            for n in prompts:
                ids = torch.randint(0, 1000, (n,), generator=gen, device="cuda", dtype=torch.int64)
                prefill(ids)
                stream.synchronize()
                reps = 5
                e0.record(stream)
                for _ in range(reps):
                    prefill(ids)
                e1.record(stream)
                stream.synchronize()
                out[n] = e0.elapsed_time(e1) / reps
            step()
            stream.synchronize()
            graph = torch.cuda.CUDAGraph()
            with torch.cuda.graph(graph, stream=stream):
                step()
            prepare(ids)
            graph.replay()
            stream.synchronize()
            e0.record(stream)
            for _ in range(n_new):
                graph.replay()
            e1.record(stream)
            stream.synchronize()
            out["decode"] = e0.elapsed_time(e1) / n_new
        return out

    rows = {}
    makers = {"layered": layered_model, "lesarax": lesarax_model}
    models = ("lesarax", "layered") if args.lesarax else ("layered", "w4a32")
    if args.layered_only != "both":
        models = tuple(m for m in models if m == args.layered_only)
    for name in (args.lesarax or args.layered).split(","):
        size = LAYERED_SIZES[name]
        W, H, G, F, L, V = size
        row = {"size": dict(zip(("hidden", "heads", "kv_heads", "ff", "layers", "vocab"), size))}
        for kind in (m for m in models if m in makers):
            cfg, w, matrix = makers[kind](torch, size, gen)
            dec = pkg.LayeredDecoder(cfg, w, "bfloat16", max_seq=max_seq, max_batch_tokens=max(prompts))
            del w
            st = dec.new_state()
            t = measure(lambda ids: dec.prefill(st, ids), lambda: dec.step(st), lambda ids: dec.prefill(st, ids))
            body = matrix - V * W
            row[kind] = {
                **{f"prefill_ms_{n}": round(t[n], 3) for n in prompts},
                **{f"prefill_tokens_per_s_{n}": round(n / t[n] * 1e3) for n in prompts},
                # matrix products alone, against the dense bf16 peak
                **{f"prefill_matrix_TFLOPs_{n}": round(2e-9 * n * body / t[n], 1) for n in prompts},
                "decode_ms": round(t["decode"], 4), "decode_tokens_per_s": round(1e3 / t["decode"], 1),
                "decode_weight_bytes": 2 * matrix, "decode_GBps": round(2e-6 * matrix / t["decode"], 1)}
            del dec, st
        if "w4a32" in models:
            shapes = {"q": (W, H * 128), "k": (W, G * 128), "v": (W, G * 128), "o": (H * 128, W), "gate": (W, F),
                      "up": (W, F), "down": (F, W)}
            pack = lambda K, N: pkg.quant_pack_rhs(torch.randn((N, K), generator=gen, device="cuda") * 0.02)
            layers = [{**{n: pack(K, N) for n, (K, N) in shapes.items()},
                       "attn_norm": torch.ones(W, device="cuda"), "ffn_norm": torch.ones(W, device="cuda")}
                      for _ in range(L)]
            emb = torch.randn((V, W), generator=gen, device="cuda")
            dec = pkg.Decoder(W, H, G, F, V, layers, emb, torch.ones(W, device="cuda"), pack(W, V), max_seq=max_seq,
                              max_batch_tokens=max(prompts))
            t = measure(lambda ids: dec.prefill(ids), lambda: dec.step(), lambda ids: dec.prefill(ids))
            body = L * sum(K * N for K, N in shapes.values())
            nbytes = L * sum(algorithmic_bytes(1, K, N, False) for K, N in shapes.values())
            nbytes += algorithmic_bytes(1, W, V, False)
            row["w4a32"] = {
                **{f"prefill_ms_{n}": round(t[n], 3) for n in prompts},
                **{f"prefill_tokens_per_s_{n}": round(n / t[n] * 1e3) for n in prompts},
                **{f"prefill_matrix_TFLOPs_{n}": round(2e-9 * n * body / t[n], 1) for n in prompts},
                "decode_ms": round(t["decode"], 4), "decode_tokens_per_s": round(1e3 / t["decode"], 1),
                "decode_weight_bytes": nbytes, "decode_GBps": round(1e-6 * nbytes / t["decode"], 1)}
            del dec, layers, emb
        torch.cuda.empty_cache()
        rows[name] = row
        print(f"# {name}: {json.dumps(row)}", file=sys.stderr, flush=True)
    title = "Lesarax beside the layered decoder" if args.lesarax else "layered decoder beside the W4A32 decoder"
    print(json.dumps({"metric": title, "unit": "ms, tokens/s", "n_gpus": 1,
                      "data": "synthetic", "dtype": "bf16" if args.lesarax else "bf16 (layered), W4A32 (w4a32)", "prompt_for_decode": max(prompts),
                      "decode_steps": n_new, "sizes": rows}))


class Linear:
    def __init__(self, pkg, torch, name, K, N, bias, gen):
        w = torch.randn((N, K), generator=gen, device="cuda", dtype=torch.float32) * 0.02
        b = (torch.randn((N,), generator=gen, device="cuda", dtype=torch.float32) * 0.02) if bias else None
        self.name, self.K, self.N, self.has_bias = name, K, N, bias
        self.packed = pkg.quant_pack_rhs(w, b)
        self.bytes = {m: algorithmic_bytes(m, K, N, bias) for m in (1, 512)}
        torch.cuda.synchronize()
        del w


def main():
    args = parse()
    if args.gpus != 1:
        print("bench.py: this build runs on ONE GPU (--gpus 1); nothing here shards across "
              "devices, so no multi-GPU figure is produced.", file=sys.stderr)
        sys.exit(2)

    import torch

    pkg = importlib.import_module("mllm-advanced_amd")
    L = pkg.lib()                       # raises if the HIP library is missing: no fallback
    assert torch.cuda.is_available(), "bench.py needs the MI355X"
    torch.cuda.set_device(0)
    if args.layered or args.lesarax:
        return layered_bench(args, torch, pkg)
    gen = torch.Generator(device="cuda")
    gen.manual_seed(0)

    # ---- synthetic model: random-init weights of the named shapes, quantised by the library
    layers = [[Linear(pkg, torch, n, K, N, b, gen) for (n, K, N, b) in LAYER_LINEARS]
              for _ in range(LAYERS)]
    lm_head = Linear(pkg, torch, *LM_HEAD, gen)
    step_linears = [lin for layer in layers for lin in layer] + [lm_head]
    step_bytes = sum(l.bytes[1] for l in step_linears)

    xgen = torch.Generator(device="cuda")
    xgen.manual_seed(1)
    x_by_k = {K: torch.randn((1, K), generator=xgen, device="cuda") for K in (1536, 8960)}
    ws_by_k = {K: torch.empty(pkg.workspace_bytes(1, K), dtype=torch.uint8, device="cuda")
               for K in (1536, 8960)}
    y_by_n = {N: torch.empty((1, N), device="cuda") for N in (256, 1536, 8960, 151936)}
    stream = torch.cuda.Stream()
    sptr = stream.cuda_stream

    def whole_op_pass():
        for l in step_linears:
            rc = L.w4a32_matmul(y_by_n[l.N].data_ptr(), x_by_k[l.K].data_ptr(), l.packed.data_ptr(),
                                ws_by_k[l.K].data_ptr(), 1, l.K, l.N, sptr)
            if rc:
                raise pkg.W4A32Error(f"w4a32_matmul({l.name}) -> {rc}")

    # The same pass as the decoder issues it: Linears that take the same input go out together
    # (q,k,v on the attention input; gate,up on the MLP input), the others alone.
    import ctypes
    y_extra = {("k", 256): torch.empty((1, 256), device="cuda"), ("up", 8960): torch.empty((1, 8960), device="cuda")}

    def group_args(lins, ys):
        cnt = len(lins)
        return ((ctypes.c_void_p * cnt)(*[t.data_ptr() for t in ys]),
                (ctypes.c_void_p * cnt)(*[l.packed.data_ptr() for l in lins]),
                (ctypes.c_int * cnt)(*[l.N for l in lins]), cnt)

    grouped_calls = []
    for layer in layers:
        q, k, v, o, gate, up, down = layer
        grouped_calls.append((group_args([q, k, v], [y_by_n[1536], y_by_n[256], y_extra[("k", 256)]]), 1536))
        grouped_calls.append((group_args([o], [y_by_n[1536]]), 1536))
        grouped_calls.append((group_args([gate, up], [y_by_n[8960], y_extra[("up", 8960)]]), 1536))
        grouped_calls.append((group_args([down], [y_by_n[1536]]), 8960))
    grouped_calls.append((group_args([lm_head], [y_by_n[151936]]), 1536))

    def grouped_pass():
        for (ya, pa, na, cnt), K in grouped_calls:
            rc = L.w4a32_matmul_grouped(ya, x_by_k[K].data_ptr(), pa, na, cnt, ws_by_k[K].data_ptr(), 1, K, sptr)
            if rc:
                raise pkg.W4A32Error(f"w4a32_matmul_grouped -> {rc}")

    # The pass with down_proj split over K: its 96 tile rows alone occupy 96 of the 256 CUs, so each tile row's
    # k range goes to several (two) workgroups, which leave partial rows; the launch that reads them (the next
    # layer's q,k,v) adds them up while it loads its row. Same Linears, same bytes, same number of launches.
    kparts = int(L.w4a32_decode_kparts(8960, 1536))
    parts_buf = torch.randn((3, 1536), generator=xgen, device="cuda") * 0.5
    parts_calls = []
    if kparts > 1:
        for li, layer in enumerate(layers):
            q, k, v, o, gate, up, down = layer
            a = pkg.DecodeLinearArgs()
            a.d_x, a.K, a.count, a.in_parts = parts_buf.data_ptr(), 1536, 3, kparts
            for i, (lin, yt) in enumerate(zip((q, k, v), (y_by_n[1536], y_by_n[256], y_extra[("k", 256)]))):
                a.d_packed[i], a.N[i], a.d_y[i] = lin.packed.data_ptr(), lin.N, yt.data_ptr()
            parts_calls.append(("decode", a))
            parts_calls.append(("grouped", grouped_calls[4 * li + 1]))
            parts_calls.append(("grouped", grouped_calls[4 * li + 2]))
            d = pkg.DecodeLinearArgs()
            d.d_x, d.K, d.count, d.out_parts = x_by_k[8960].data_ptr(), 8960, 1, kparts
            d.d_packed[0], d.N[0], d.d_y[0] = down.packed.data_ptr(), 1536, parts_buf.data_ptr()
            parts_calls.append(("decode", d))
        parts_calls.append(("grouped", grouped_calls[-1]))

    def parts_pass():
        for kind, c in parts_calls:
            if kind == "decode":
                rc = L.w4a32_decode_linear(ctypes.byref(c), sptr)
            else:
                (ya, pa, na, cnt), K = c
                rc = L.w4a32_matmul_grouped(ya, x_by_k[K].data_ptr(), pa, na, cnt, ws_by_k[K].data_ptr(), 1, K, sptr)
            if rc:
                raise pkg.W4A32Error(f"parts pass ({kind}) -> {rc}")

    def product_only_pass():
        for l in step_linears:
            rc = L.w4a32_matmul_quantized(y_by_n[l.N].data_ptr(), ws_by_k[l.K].data_ptr(),
                                          l.packed.data_ptr(), 1, l.K, l.N, sptr)
            if rc:
                raise pkg.W4A32Error(f"w4a32_matmul_quantized({l.name}) -> {rc}")

    def timed(fn, steps, warmup, use_graph):
        """warmup, then exactly `steps` passes between two events on the launch stream."""
        with torch.cuda.stream(stream):
            for _ in range(max(warmup, 1)):
                fn()
            stream.synchronize()
            run = fn
            if use_graph:
                graph = torch.cuda.CUDAGraph()
                with torch.cuda.graph(graph, stream=stream):
                    fn()
                run = graph.replay
                run()
                stream.synchronize()
            e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            e0.record(stream)
            for _ in range(steps):
                run()
            e1.record(stream)
            torch.cuda.synchronize()
            wall = time.perf_counter() - t0
        return e0.elapsed_time(e1) / steps, wall * 1e3 / steps

    use_graph = not args.eager

    if args.traffic_probe:
        # known traffic first: 256 MiB read + 256 MiB written by a plain copy kernel
        src = torch.empty(256 << 20, dtype=torch.uint8, device="cuda").fill_(1)
        dst = torch.empty_like(src)
        with torch.cuda.stream(stream):
            for _ in range(3):
                dst.copy_(src)
            gate, M = layers[0][4], 512
            # three different gate_proj buffers (cold weights each time), then lm_head three times
            for lin in (layers[1][4], layers[2][4], layers[3][4], lm_head, lm_head, lm_head):
                L.w4a32_matmul(y_by_n[lin.N].data_ptr(), x_by_k[lin.K].data_ptr(),
                               lin.packed.data_ptr(), ws_by_k[lin.K].data_ptr(), 1, lin.K, lin.N, sptr)
            x = torch.randn((M, gate.K), generator=xgen, device="cuda")
            ws = torch.empty(pkg.workspace_bytes(M, gate.K), dtype=torch.uint8, device="cuda")
            y = torch.empty((M, gate.N), device="cuda")
            for _ in range(3):
                L.w4a32_matmul(y.data_ptr(), x.data_ptr(), gate.packed.data_ptr(), ws.data_ptr(), M,
                               gate.K, gate.N, sptr)
            # down_proj (K = 8960) at M = 512 through the 128 x 64 tile shape, plain kernel: 96 workgroups,
            # each alone on its CU, 140 stages each (the launch whose instruction counters are profiled)
            down = layers[0][6]
            xd = torch.randn((M, down.K), generator=xgen, device="cuda")
            wsd = torch.empty(pkg.workspace_bytes(M, down.K), dtype=torch.uint8, device="cuda")
            yd = torch.empty((M, down.N), device="cuda")
            L.w4a32_quant_lhs(xd.data_ptr(), M, down.K, down.K, wsd.data_ptr(), sptr)
            for _ in range(3):
                L.w4a32_matmul_quantized_ex(yd.data_ptr(), wsd.data_ptr(), down.packed.data_ptr(), M, down.K,
                                            down.N, pkg.KERNEL_GEMM_F16_TILE0 + 4, sptr)
        torch.cuda.synchronize()
        print(json.dumps({"traffic_probe": {
            "copy_bytes_read": 256 << 20, "copy_bytes_written": 256 << 20,
            "gate_proj_M1_algorithmic_bytes": gate.bytes[1], "lm_head_M1_algorithmic_bytes": lm_head.bytes[1],
            "gate_proj_M512_weight_bytes": gate.bytes[1] - 1 * gate.K * 4 - 1 * gate.N * 4}}))
        return

    # Every call is ONE kernel (row quantisation inside): gemv_fused_kernel for the decoder
    # Linears (q,k,v in one launch, gate,up in one launch), gemv_wide_kernel for lm_head.
    ms_unsplit = ms_parts = None
    if args.which_pass != "split" or not parts_calls:
        ms_unsplit, wall_unsplit = timed(grouped_pass, args.steps, args.warmup, use_graph)
        ms_step, wall_ms, split_down = ms_unsplit, wall_unsplit, False
    if parts_calls and args.which_pass != "unsplit":
        ms_parts, wall_parts = timed(parts_pass, args.steps, args.warmup, use_graph)
        if ms_unsplit is None or ms_parts < ms_unsplit:
            ms_step, wall_ms, split_down = ms_parts, wall_parts, True
    n_launch = len(grouped_calls)
    roof_avg_us = ms_step * 1e3 / n_launch
    roof_bytes = step_bytes / n_launch
    achieved = roof_bytes / (roof_avg_us * 1e-6) / 1e9
    roofline = {"bound": "hbm", "achieved": round(achieved, 1), "peak": HBM_PEAK_GBS, "unit": "GB/s",
                "frac": round(achieved / HBM_PEAK_GBS, 4), "traffic": PASS_TRAFFIC_BYTES_PER_LAUNCH,
                "traffic_source": "rocprofv3 --pmc FETCH_SIZE / WRITE_SIZE over this pass's 113 launches "
                                  "(3893.2 / 29.1 KiB per dispatch), scaled x2.00 / x1.00 by the same counters' "
                                  "reading for a 256 MiB copy; profiles/traffic_fetch_write_decode_prefill.md",
                "kernel": "gemv_fused_kernel<1,1> for K=1536 (q,k,v grouped; o; gate,up as a pair), "
                          "gemv_kparts_kernel<2> for down_proj (K=8960 in two k-parts; gemv_fused_kernel<1,2> "
                          "when the unsplit pass is the faster one), gemv_wide_kernel<1,true> for lm_head",
                "launches_per_step": n_launch, "avg_launch_us": round(roof_avg_us, 3),
                "algorithmic_bytes_per_launch": int(roof_bytes),
                "note": "average over the step's 113 launches (28 x {qkv, o, gate+up, down} + lm_head), "
                        "launch period inside a HIP graph; per-shape figures are in extra"}
    if args.roofline_only:
        print(json.dumps({"roofline": roofline}))
        return

    value = step_bytes / (ms_step * 1e-3) / 1e9
    # the same Linears one launch each (what the per-op boundary does without grouping) ...
    ms_single, _ = timed(whole_op_pass, args.steps, args.warmup, use_graph)
    # ... and the products alone on activations quantised once
    with torch.cuda.stream(stream):
        for K in ws_by_k:
            L.w4a32_quant_lhs(x_by_k[K].data_ptr(), 1, K, K, ws_by_k[K].data_ptr(), sptr)
    stream.synchronize()
    ms_prod, _ = timed(product_only_pass, args.steps, args.warmup, use_graph)

    extra = {"decode_linears_tokens_per_s": round(1e3 / ms_step, 1),
             "down_proj_split_over_k": {"used_for_value": split_down, "parts": kparts,
                                        "ms_per_step_unsplit": None if ms_unsplit is None else round(ms_unsplit, 4),
                                        "ms_per_step_split": None if ms_parts is None else round(ms_parts, 4)},
             "wall_ms_per_step": round(wall_ms, 4), "graph": use_graph,
             "one_launch_per_linear": {"launches": len(step_linears), "ms_per_step": round(ms_single, 4),
                                       "GBps": round(step_bytes / (ms_single * 1e-3) / 1e9, 1)},
             "product_only_ms_per_step": round(ms_prod, 4)}

    # ---- the same pass on 4 and 8 rows (batched decode): same launches, same weight bytes
    batched = {}
    for Mb in (4, 8):
        xb = {K: torch.randn((Mb, K), generator=xgen, device="cuda") for K in (1536, 8960)}
        wsb = {K: torch.empty(pkg.workspace_bytes(Mb, K), dtype=torch.uint8, device="cuda")
               for K in (1536, 8960)}
        yb = {N: torch.empty((Mb, N), device="cuda") for N in (256, 1536, 8960, 151936)}
        yb2 = {256: torch.empty((Mb, 256), device="cuda"), 8960: torch.empty((Mb, 8960), device="cuda")}
        calls_b = []
        for layer in layers:
            q, k, v, o, gate, up, down = layer
            calls_b.append((group_args([q, k, v], [yb[1536], yb[256], yb2[256]]), 1536))
            calls_b.append((group_args([o], [yb[1536]]), 1536))
            calls_b.append((group_args([gate, up], [yb[8960], yb2[8960]]), 1536))
            calls_b.append((group_args([down], [yb[1536]]), 8960))
        calls_b.append((group_args([lm_head], [yb[151936]]), 1536))

        def batched_pass(calls_b=calls_b, xb=xb, wsb=wsb, Mb=Mb):
            for (ya, pa, na, cnt), K in calls_b:
                rc = L.w4a32_matmul_grouped(ya, xb[K].data_ptr(), pa, na, cnt, wsb[K].data_ptr(), Mb, K, sptr)
                if rc:
                    raise pkg.W4A32Error(f"w4a32_matmul_grouped M={Mb} -> {rc}")
        ms_b, _ = timed(batched_pass, args.steps, args.warmup, use_graph)
        bytes_b = sum(algorithmic_bytes(Mb, l.K, l.N, l.has_bias) for l in step_linears)
        # the pass's launches kind by kind (a graph of the 28 launches of one kind, lm_head: 28 launches over
        # three copies of its weights), so that the pass's time is attributable at this M as well
        kinds_b = {}
        lm_copies = [lm_head] + [Linear(pkg, torch, *LM_HEAD, gen) for _ in range(2)]
        kind_calls = {"q,k,v grouped": calls_b[0:4 * LAYERS:4], "o_proj": calls_b[1:4 * LAYERS:4],
                      "gate,up grouped": calls_b[2:4 * LAYERS:4], "down_proj": calls_b[3:4 * LAYERS:4],
                      "lm_head": [(group_args([lm_copies[i % 3]], [yb[151936]]), 1536) for i in range(27)]}
        for label, kc in kind_calls.items():
            def kind_pass(kc=kc, xb=xb, wsb=wsb, Mb=Mb):
                for (ya, pa, na, cnt), K in kc:
                    rc = L.w4a32_matmul_grouped(ya, xb[K].data_ptr(), pa, na, cnt, wsb[K].data_ptr(), Mb, K, sptr)
                    if rc:
                        raise pkg.W4A32Error(f"w4a32_matmul_grouped M={Mb} ({label}) -> {rc}")
            ms_k, _ = timed(kind_pass, 10, 2, use_graph)
            kinds_b[label] = {"us": round(ms_k * 1e3 / len(kc), 2), "launches_per_step": 1 if label == "lm_head" else LAYERS}
        kinds_b["sum_us"] = round(sum(v["us"] * v["launches_per_step"] for v in kinds_b.values()), 1)
        del lm_copies
        batched[f"M{Mb}"] = {"ms_per_step": round(ms_b, 4), "GBps": round(bytes_b / (ms_b * 1e-3) / 1e9, 1),
                             "rows_per_s": round(Mb * 1e3 / ms_b, 1),
                             "flop_equiv_TFLOPs": round(sum(2.0 * Mb * l.K * l.N for l in step_linears)
                                                        / (ms_b * 1e-3) / 1e12, 2),
                             "by_kernel": kinds_b}
    extra["decode_pass_batched"] = batched

    # ---- per-shape decode figures (product kernel, weights rotated over the 28 layers)
    per_shape = {}
    reps = 20
    with torch.cuda.stream(stream):
        for idx, (name, K, N, b) in enumerate(LAYER_LINEARS + [LM_HEAD]):
            if name == "lm_head":
                # three copies, 396 MB in all, so that no repetition finds its weights in the
                # 256 MB Infinity Cache
                lins = [lm_head] + [Linear(pkg, torch, *LM_HEAD, gen) for _ in range(2)]
            else:
                lins = [layer[idx] for layer in layers]
            e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)

            def one_round(lins=lins, K=K, N=N):
                for l in lins:
                    L.w4a32_matmul(y_by_n[N].data_ptr(), x_by_k[K].data_ptr(), l.packed.data_ptr(),
                                   ws_by_k[K].data_ptr(), 1, K, N, sptr)
            one_round()
            stream.synchronize()
            run = one_round
            if use_graph:      # as in the step: launch period on the device, not the host's call rate
                g_shape = torch.cuda.CUDAGraph()
                with torch.cuda.graph(g_shape, stream=stream):
                    one_round()
                run = g_shape.replay
                run()
            e0.record(stream)
            for _ in range(reps):
                run()
            e1.record(stream)
            stream.synchronize()
            us = e0.elapsed_time(e1) * 1e3 / (reps * len(lins))
            gbs = lins[0].bytes[1] / (us * 1e-6) / 1e9
            per_shape[name] = {"us": round(us, 2), "GBps": round(gbs, 1),
                               "frac_of_hbm_peak": round(gbs / HBM_PEAK_GBS, 3),
                               "note": ("rotating over 3 weight buffers (396 MB)"
                                        if name == "lm_head" else "rotating over 28 weight buffers")}
    extra["decode_per_shape"] = per_shape

    # ---- the pass's own launches, kind by kind (28 launches of one kind, each on its layer's weights,
    # replayed from a graph like the pass): un-profiled launch periods whose sum is the pass
    by_kernel = {}
    kinds = [("q,k,v grouped", 0, ["q_proj", "k_proj", "v_proj"]), ("o_proj", 1, ["o_proj"]),
             ("gate,up grouped", 2, ["gate_proj", "up_proj"]), ("down_proj", 3, ["down_proj"])]
    name_bytes = {l.name: l.bytes[1] for l in layers[0]}
    with torch.cuda.stream(stream):
        for label, slot, names in kinds:
            if split_down and slot in (0, 3):     # the launches the pass is made of: the split forms
                calls = [parts_calls[4 * i + slot] for i in range(LAYERS)]
                label += f" (reads {kparts} partial rows)" if slot == 0 else f" (k range in {kparts} parts)"
            else:
                calls = [("grouped", grouped_calls[4 * i + slot]) for i in range(LAYERS)]

            def kind_round(calls=calls):
                for kind, c in calls:
                    if kind == "decode":
                        L.w4a32_decode_linear(ctypes.byref(c), sptr)
                    else:
                        (ya, pa, na, cnt), K = c
                        L.w4a32_matmul_grouped(ya, x_by_k[K].data_ptr(), pa, na, cnt, ws_by_k[K].data_ptr(), 1, K, sptr)
            kind_round()
            stream.synchronize()
            run = kind_round
            if use_graph:
                g_kind = torch.cuda.CUDAGraph()
                with torch.cuda.graph(g_kind, stream=stream):
                    kind_round()
                run = g_kind.replay
                run()
            e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            e0.record(stream)
            for _ in range(reps):
                run()
            e1.record(stream)
            stream.synchronize()
            us = e0.elapsed_time(e1) * 1e3 / (reps * LAYERS)
            # the input row is read once per launch, not once per Linear
            nbytes = sum(name_bytes[n] for n in names) - (len(names) - 1) * 1536 * 4
            by_kernel[label] = {"launches_per_step": LAYERS, "us": round(us, 2), "bytes": nbytes,
                                "GBps": round(nbytes / (us * 1e-6) / 1e9, 1),
                                "frac_of_hbm_peak": round(nbytes / (us * 1e-6) / 1e9 / HBM_PEAK_GBS, 3)}
    by_kernel["lm_head"] = {"launches_per_step": 1, "us": per_shape["lm_head"]["us"], "bytes": lm_head.bytes[1],
                            "GBps": per_shape["lm_head"]["GBps"],
                            "frac_of_hbm_peak": per_shape["lm_head"]["frac_of_hbm_peak"]}
    by_kernel["sum_us"] = round(sum(v["us"] * v["launches_per_step"] for v in by_kernel.values()), 1)
    by_kernel["step_us"] = round(ms_step * 1e3, 1)
    by_kernel["note"] = ("launch periods measured by events on the launch stream without a profiler, each kind "
                         "in a graph of its 28 launches; sum_us is what they add up to per step, step_us the "
                         "step as timed (rocprofv3's per-kernel durations of the same launches, which exclude "
                         "the gap between kernels but carry the profiler's own cost, are in profiles/)")
    extra["roofline_by_kernel"] = by_kernel

    # ---- prefill leg: whole op (row quant + product) and the product kernel alone
    if not args.no_gemm:
        prefill = {}
        with torch.cuda.stream(stream):
            for M in (128, 512, 2048):
                per, tot_flop, tot_ms, tot_kms = {}, 0.0, 0.0, 0.0
                for idx, (name, K, N, b) in enumerate(LAYER_LINEARS):
                    lin = layers[0][idx]
                    x = torch.randn((M, K), generator=xgen, device="cuda")
                    x[: max(1, M // 100)] *= 20.0      # 1 % of rows x20: per-row scales matter
                    # sized for the whole-op call that may deal a long k range to several workgroups itself
                    ws = torch.empty(int(L.w4a32_workspace_bytes_n(M, K, N)), dtype=torch.uint8, device="cuda")
                    y = torch.empty((M, N), device="cuda")

                    def whole():
                        rc = L.w4a32_matmul_ws(y.data_ptr(), x.data_ptr(), lin.packed.data_ptr(),
                                               ws.data_ptr(), ws.numel(), M, K, N, sptr)
                        if rc:
                            raise pkg.W4A32Error(f"w4a32_matmul_ws M={M} ({name}) -> {rc}")

                    def kernel_only():
                        rc = L.w4a32_matmul_quantized(y.data_ptr(), ws.data_ptr(), lin.packed.data_ptr(),
                                                      M, K, N, sptr)
                        if rc:
                            raise pkg.W4A32Error(f"w4a32_matmul_quantized M={M} ({name}) -> {rc}")
                    times = []
                    for fn in (whole, kernel_only):
                        for _ in range(3):
                            fn()
                        e0 = torch.cuda.Event(enable_timing=True)
                        e1 = torch.cuda.Event(enable_timing=True)
                        e0.record(stream)
                        for _ in range(20):
                            fn()
                        e1.record(stream)
                        stream.synchronize()
                        times.append(e0.elapsed_time(e1) / 20)
                    flop = 2.0 * M * N * K
                    per[name] = {"ms": round(times[0], 4), "TFLOPs": round(flop / (times[0] * 1e-3) / 1e12, 1),
                                 "kernel_ms": round(times[1], 4),
                                 "kernel_TFLOPs": round(flop / (times[1] * 1e-3) / 1e12, 1)}
                    tot_flop += flop
                    tot_ms += times[0]
                    tot_kms += times[1]
                # The layer's Linears as a prefill issues them: rows quantised once per input, q,k,v as one
                # grouped launch, gate,up as one launch that stores silu(gate) * up only, down with its k
                # range split over workgroups (partial sums in lent scratch).
                lay = layers[0]
                xh = torch.randn((M, 1536), generator=xgen, device="cuda")
                xi = torch.randn((M, 8960), generator=xgen, device="cuda")
                ws_h = torch.empty(pkg.workspace_bytes(M, 1536), dtype=torch.uint8, device="cuda")
                ws_i = torch.empty(pkg.workspace_bytes(M, 8960), dtype=torch.uint8, device="cuda")
                yq, yk, yv = (torch.empty((M, n), device="cuda") for n in (1536, 256, 256))
                yg = torch.empty((M, 8960), device="cuda")
                yo = torch.empty((M, 1536), device="cuda")
                scratch = torch.empty(max(16, int(L.w4a32_splitk_scratch_bytes(M, 8960, 1536))),
                                      dtype=torch.uint8, device="cuda")

                def issued():
                    pkg.quant_lhs(xh, ws_h)
                    pkg.matmul_quantized_grouped(ws_h, [lay[0].packed, lay[1].packed, lay[2].packed],
                                                 [1536, 256, 256], M, 1536, outs=[yq, yk, yv])
                    pkg.quant_lhs(xh, ws_h)
                    pkg.matmul_quantized(ws_h, lay[3].packed, M, 1536, 1536, out=yo)
                    pkg.quant_lhs(xh, ws_h)
                    pkg.matmul_quantized_silu_pair(ws_h, lay[4].packed, lay[5].packed, M, 1536, 8960, out=yg)
                    pkg.quant_lhs(xi, ws_i)
                    pkg.matmul_quantized_splitk(ws_i, lay[6].packed, M, 8960, 1536, scratch=scratch, out=yo)
                for _ in range(3):
                    issued()
                e0 = torch.cuda.Event(enable_timing=True)
                e1 = torch.cuda.Event(enable_timing=True)
                e0.record(stream)
                for _ in range(20):
                    issued()
                e1.record(stream)
                stream.synchronize()
                issued_ms = e0.elapsed_time(e1) / 20
                prefill[f"M{M}"] = {"per_shape": per,
                                    "layer_TFLOPs": round(tot_flop / (tot_ms * 1e-3) / 1e12, 1),
                                    "layer_kernel_TFLOPs": round(tot_flop / (tot_kms * 1e-3) / 1e12, 1),
                                    "layer_as_issued_ms": round(issued_ms, 4),
                                    "layer_as_issued_TFLOPs": round(tot_flop / (issued_ms * 1e-3) / 1e12, 1)}
        extra["prefill"] = prefill
        best = prefill["M2048"]["per_shape"]["gate_proj"]["kernel_TFLOPs"]
        # the same kernel with many tiles per CU (beyond the configurations' sizes: what the kernel sustains)
        with torch.cuda.stream(stream):
            Mbig, (_, Kb, Nb, _) = 8192, LAYER_LINEARS[4]
            xb_ = torch.randn((Mbig, Kb), generator=xgen, device="cuda")
            wsb_ = pkg.quant_lhs(xb_)
            yb_ = torch.empty((Mbig, Nb), device="cuda")
            for _ in range(3):
                L.w4a32_matmul_quantized(yb_.data_ptr(), wsb_.data_ptr(), layers[0][4].packed.data_ptr(), Mbig,
                                         Kb, Nb, sptr)
            e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            e0.record(stream)
            for _ in range(10):
                L.w4a32_matmul_quantized(yb_.data_ptr(), wsb_.data_ptr(), layers[0][4].packed.data_ptr(), Mbig,
                                         Kb, Nb, sptr)
            e1.record(stream)
            stream.synchronize()
            big_tflops = 2.0 * Mbig * Nb * Kb / (e0.elapsed_time(e1) / 10 * 1e-3) / 1e12
            del xb_, wsb_, yb_
        g512 = prefill["M512"]["per_shape"]["gate_proj"]
        extra["prefill_roofline"] = {
            "bound": "mfma", "kernel": "gemm_f16_kernel (v_mfma_f32_32x32x16_f16)",
            "workload": "gate_proj M=512 K=1536 N=8960 (the configuration the GEMM metric names), product "
                        "kernel alone; whole_op adds the row quantiser that the reference's Linear includes",
            "achieved": g512["kernel_TFLOPs"], "peak": 2500.0, "unit": "TFLOP/s",
            "frac": round(g512["kernel_TFLOPs"] / 2500.0, 4),
            "whole_op": {"achieved": g512["TFLOPs"], "frac": round(g512["TFLOPs"] / 2500.0, 4)},
            "layer_as_issued_M512": {"achieved": prefill["M512"]["layer_as_issued_TFLOPs"],
                                     "frac": round(prefill["M512"]["layer_as_issued_TFLOPs"] / 2500.0, 4)},
            "other_M": {"M2048_gate_proj_kernel": {"achieved": best, "frac": round(best / 2500.0, 4)},
                        "M2048_gate_proj_whole_op": {
                            "achieved": prefill["M2048"]["per_shape"]["gate_proj"]["TFLOPs"],
                            "frac": round(prefill["M2048"]["per_shape"]["gate_proj"]["TFLOPs"] / 2500.0, 4)},
                        "M8192_gate_proj_kernel": {"achieved": round(big_tflops, 1),
                                                   "frac": round(big_tflops / 2500.0, 4)}},
            "M512_gate_proj_kernel_TFLOPs": g512["kernel_TFLOPs"]}

    # ---- config 4: the whole decoder (same Linears plus the f32 operators between them), batch 1,
    # 512-token random-id prompt, then 256 greedy steps replayed from one captured HIP graph
    if not args.no_decoder:
        H, V, I = 1536, 151936, 8960
        dgen = torch.Generator(device="cuda")
        dgen.manual_seed(2)
        emb = torch.randn((V, H), generator=dgen, device="cuda")
        norm = lambda: 1 + 0.1 * torch.randn((H,), generator=dgen, device="cuda")
        dl = []
        for layer in layers:
            d = {n: lin.packed for n, lin in zip(("q", "k", "v", "o", "gate", "up", "down"), layer)}
            d["attn_norm"], d["ffn_norm"] = norm(), norm()
            dl.append(d)
        with torch.cuda.stream(stream):
            dec = pkg.Decoder(H, 12, 2, I, V, dl, emb, norm(), lm_head.packed, max_seq=1024,
                              max_batch_tokens=512, rope_theta=1e6, rms_eps=1e-6)
            prompt = torch.randint(0, V, (512,), generator=dgen, device="cuda", dtype=torch.int64)
            dec.prefill(prompt)                      # warm-up (allocations, code objects)
            stream.synchronize()
            e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            e0.record(stream)
            for _ in range(3):
                dec.prefill(prompt)
            e1.record(stream)
            stream.synchronize()
            prefill_ms = e0.elapsed_time(e1) / 3
            first = int(dec.token)
            dec.step()                               # warm-up of the step, then rewind by prefilling again
            dec.prefill(prompt)
            graph = torch.cuda.CUDAGraph()
            with torch.cuda.graph(graph, stream=stream):
                dec.step()
            stream.synchronize()
            n_new = 256
            e0.record(stream)
            for _ in range(n_new):
                graph.replay()
            e1.record(stream)
            stream.synchronize()
            decode_ms = e0.elapsed_time(e1)
            # the timed tokens are real: the position advanced once per replay, the last step's logits are
            # finite and its token is the first maximum of those logits
            logits = dec.logits
            assert dec.position == 512 + n_new
            assert bool(torch.isfinite(logits).all()), "decoder produced non-finite logits"
            assert int(dec.token) == int(torch.argmax(logits)), "token is not the argmax of the logits"
            assert 0 <= first < V
        extra["decoder_config4"] = {
            "workload": "28 layers, hidden 1536, 12 q / 2 kv heads x 128, MLP 8960, vocab 151936, rope theta 1e6, "
                        "f32 KV cache; batch 1, 512 random prompt ids (prefill: mean of 3 runs), 256 greedy steps; "
                        "all Linears W4A32 (lm_head included), random-init weights",
            "prefill_ms_512_tokens": round(prefill_ms, 2),
            "prefill_tokens_per_s": round(512 / (prefill_ms * 1e-3), 1),
            "decode_ms_per_token": round(decode_ms / n_new, 4),
            "decode_tokens_per_s": round(n_new / (decode_ms * 1e-3), 1),
            "decode_weight_GBps": round(step_bytes / (decode_ms / n_new * 1e-3) / 1e9, 1),
            "note": "one decode step = 142 launches (28 x [add+norm+qkv (layer 0: on the token's embedding row, "
                    "gathered), rope+cache+attention slices, o merging the slices, add+norm+gate/up+silu*mul, down "
                    "in two k-parts], add+norm+lm_head, argmax over lm_head's partial results), captured once and "
                    "replayed; positions and cache lengths are read from device memory",
        }
        # the same decoder with lm_head as the reference's W4A32 quantizer configuration stores it: a dense Fp16
        # [V][H] matrix applied as a plain matmul (466.7 MB per token instead of the W4A32 head's 131.9 MB)
        with torch.cuda.stream(stream):
            head16 = (torch.randn((V, H), generator=dgen, device="cuda") * 0.02).half()
            dec16 = pkg.Decoder(H, 12, 2, I, V, dl, emb, norm(), head16, max_seq=1024, max_batch_tokens=512,
                                rope_theta=1e6, rms_eps=1e-6, lm_head_dense=True)
            dec16.prefill(prompt)
            dec16.step()
            dec16.prefill(prompt)
            graph16 = torch.cuda.CUDAGraph()
            with torch.cuda.graph(graph16, stream=stream):
                dec16.step()
            stream.synchronize()
            e0.record(stream)
            for _ in range(n_new):
                graph16.replay()
            e1.record(stream)
            stream.synchronize()
            dense_ms = e0.elapsed_time(e1) / n_new
            assert dec16.position == 512 + n_new
            assert int(dec16.token) == int(torch.argmax(dec16.logits)), "token is not the argmax of the logits"
            extra["decoder_config4"]["dense_f16_lm_head"] = {
                "decode_ms_per_token": round(dense_ms, 4), "decode_tokens_per_s": round(1e3 / dense_ms, 1),
                "lm_head_bytes": V * H * 2,
                "note": "lm_head as a dense Fp16 matrix (the reference's own form) instead of W4A32; the other "
                        "141 launches are the same"}
            del dec16, head16, graph16
        # config 5, language side: prefill of the 256 merged vision tokens through the same decoder
        with torch.cuda.stream(stream):
            p256 = prompt[:256].contiguous()
            dec.prefill(p256)
            stream.synchronize()
            e0.record(stream)
            dec.prefill(p256)
            e1.record(stream)
            stream.synchronize()
            lm256_ms = e0.elapsed_time(e1)
        del dec, emb

        # config 5, vision side: Qwen2-VL-2B ViT Linears at M = 1024 patch tokens (32 layers of
        # qkv 1280->3840, proj 1280->1280, fc1 1280->5120, fc2 5120->1280), the patch embedding as
        # im2col + Linear (K = 3*2*14*14 = 1176 padded to 1184, N = 1280) and the merger (5120->5120->1536
        # on 256 rows)
        vgen = torch.Generator(device="cuda")
        vgen.manual_seed(3)
        vit = {}
        with torch.cuda.stream(stream):
            def time_linear(M, K, N, reps=20):
                w = torch.randn((N, K), generator=vgen, device="cuda") * 0.02
                b = torch.randn((N,), generator=vgen, device="cuda") * 0.02
                packed = pkg.quant_pack_rhs(w, b)
                x = torch.randn((M, K), generator=vgen, device="cuda")
                ws = torch.empty(pkg.workspace_bytes(M, K), dtype=torch.uint8, device="cuda")
                y = torch.empty((M, N), device="cuda")
                for _ in range(3):
                    pkg.matmul(x, packed, N, ws=ws, out=y)
                e0.record(stream)
                for _ in range(reps):
                    pkg.matmul(x, packed, N, ws=ws, out=y)
                e1.record(stream)
                stream.synchronize()
                ms = e0.elapsed_time(e1) / reps
                return {"ms": round(ms, 4), "TFLOPs": round(2.0 * M * N * K / (ms * 1e-3) / 1e12, 1)}
            layer_ms, layer_flop = 0.0, 0.0
            for name, K, N in (("qkv", 1280, 3840), ("proj", 1280, 1280), ("fc1", 1280, 5120), ("fc2", 5120, 1280)):
                vit[name] = time_linear(1024, K, N)
                layer_ms += vit[name]["ms"]
                layer_flop += 2.0 * 1024 * N * K
            vit["merger_fc1"] = time_linear(256, 5120, 5120)
            vit["merger_fc2"] = time_linear(256, 5120, 1536)
            img = torch.randn((1, 3, 2, 448, 448), generator=vgen, device="cuda")
            wpe = torch.zeros((1280, 1184), device="cuda")
            wpe[:, :1176] = torch.randn((1280, 1176), generator=vgen, device="cuda") * 0.02
            pe_packed = pkg.quant_pack_rhs(wpe)
            for _ in range(2):
                pkg.matmul(pkg.op_im2col_conv3d(img, (2, 14, 14), (2, 14, 14)), pe_packed, 1280)
            e0.record(stream)
            for _ in range(10):
                pkg.matmul(pkg.op_im2col_conv3d(img, (2, 14, 14), (2, 14, 14)), pe_packed, 1280)
            e1.record(stream)
            stream.synchronize()
            vit["patch_embed_im2col_plus_linear_ms"] = round(e0.elapsed_time(e1) / 10, 4)
        extra["vit_config5"] = {
            "workload": "Qwen2-VL-2B-shaped vision Linears as W4A32 GEMM, 1024 patch tokens (one 448x448 image), "
                        "whole op (row quant + product) per Linear; python-side allocation of the im2col "
                        "buffer is inside the patch-embed figure",
            "per_linear_M1024": vit,
            "vit_layer_linears_ms": round(layer_ms, 4),
            "vit_32_layers_linears_ms": round(32 * layer_ms, 3),
            "vit_layer_TFLOPs": round(layer_flop / (layer_ms * 1e-3) / 1e12, 1),
            "lm_prefill_256_tokens_ms": round(lm256_ms, 3),
        }

    # ---- CPU baseline: scalar restatement of the reference path, bounded sample
    cpu = None
    if not args.no_cpu:
        sys.path.insert(0, os.path.join(ROOT, "oracle"))
        import w4a32_oracle as orc
        sample = layers[0]
        host = []
        for l in sample:
            u4, sc, bias = pkg.unpack_native(l.packed, l.N, l.K, want_bias=True)
            torch.cuda.synchronize()
            host.append((l, u4.cpu().numpy(), sc.cpu().numpy().view("uint16"),
                         bias.cpu().numpy() if l.has_bias else None))
        xs = {K: x_by_k[K].cpu().numpy() for K in x_by_k}
        for (l, u4, sc, bias) in host:      # page in
            orc.linear(xs[l.K], u4, sc, bias=bias, threads=1)
        reps_cpu, t0 = 0, time.perf_counter()
        while time.perf_counter() - t0 < 10.0:
            for (l, u4, sc, bias) in host:
                orc.linear(xs[l.K], u4, sc, bias=bias, threads=1)
            reps_cpu += 1
        dt = time.perf_counter() - t0
        layer_bytes = sum(l.bytes[1] for l in sample)
        cpu = {"value": round(layer_bytes * reps_cpu / dt / 1e9, 3), "unit": "GB/s", "cores": 1,
               "kind": "port",
               "sample": f"{reps_cpu} passes over one decoder layer's 7 W4A32 Linears at M=1 "
                         f"({layer_bytes} algorithmic bytes per pass), scalar C restatement of the "
                         f"reference path; the reference runs decode (M=1) as a single task",
               "host_cpus": os.cpu_count()}
        # the same restatement with its output columns dealt to threads (the reference itself splits rows
        # only, so it gains nothing at M=1): 4 threads = the reference's default pool, 16 = this box's share
        threaded = {}
        for nthr in (4, 16):
            reps_t, t0 = 0, time.perf_counter()
            while time.perf_counter() - t0 < 3.0:
                for (l, u4, sc, bias) in host:
                    orc.linear(xs[l.K], u4, sc, bias=bias, threads=nthr)
                reps_t += 1
            threaded[f"threads_{nthr}"] = round(layer_bytes * reps_t / (time.perf_counter() - t0) / 1e9, 3)
        # the same product with its block dots on AVX-512 VNNI (bit-identical results), where the host has it
        vnni = None
        if orc.has_vnni():
            vnni = {}
            for nthr in (1, 4, 16):
                reps_t, t0 = 0, time.perf_counter()
                while time.perf_counter() - t0 < 2.0:
                    for (l, u4, sc, bias) in host:
                        orc.linear_vnni(xs[l.K], u4, sc, bias=bias, threads=nthr)
                    reps_t += 1
                vnni[f"threads_{nthr}"] = round(layer_bytes * reps_t / (time.perf_counter() - t0) / 1e9, 3)
        # prefill: gate_proj at M=128 (the reference deals rows to its 4 workers)
        (l, u4, sc, bias) = host[4]
        xp = np.random.default_rng(1).standard_normal((128, l.K)).astype(np.float32)
        t0 = time.perf_counter()
        orc.linear(xp, u4, sc, bias=bias, threads=4)
        dtp = time.perf_counter() - t0
        # The headline block states the best the host does on this path, with the core count it took; the
        # other variants (the faithful 1-thread scalar form first) stand beside it, each with its cores.
        variants = [{"form": "scalar C restatement, one task (how the reference runs M=1, kai_linear.cpp:370)",
                     "cores": 1, "GBps": cpu["value"]}]
        variants += [{"form": "scalar C restatement, output columns dealt to OpenMP threads", "cores": int(k.split("_")[1]),
                      "GBps": v} for k, v in threaded.items()]
        if vnni:
            variants += [{"form": "AVX-512 VNNI block dots (bit-identical to the scalar form), columns dealt to "
                                  "OpenMP threads", "cores": int(k.split("_")[1]), "GBps": v} for k, v in vnni.items()]
        best = max(variants, key=lambda v: v["GBps"])
        cpu = {"value": best["GBps"], "unit": "GB/s", "cores": best["cores"], "kind": "port",
               "form": best["form"], "sample": cpu["sample"] + "; every variant runs the same sample for 2-10 s",
               "host_cpus": os.cpu_count(), "variants": variants}
        extra["cpu_baseline_more"] = {"decode_GBps_by_threads": threaded,
                                      "decode_GBps_avx512_vnni_by_threads": vnni,
                                      "prefill_gate_proj_M128_4_threads_TFLOPs":
                                          round(2.0 * 128 * l.N * l.K / dtp / 1e12, 5),
                                      "note": "scalar C restatement; columns (decode) or rows x columns "
                                              "(prefill) dealt to OpenMP threads"}

    out = {
        "metric": "W4 GEMV HBM GB/s (M=1)", "value": round(value, 1), "unit": "GB/s",
        "n_gpus": 1, "steps": args.steps, "warmup": args.warmup, "ms_per_step": round(ms_step, 4),
        "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "int8",
        "data": "synthetic (torch cuda generator seed 0, N(0,0.02^2) f32 weights quantised to 4-bit "
                "block-32 by the library; activations N(0,1) seed 1)",
        "config": {"workload": "config 2 at M=1: Qwen2-1.5B decode Linears, 28 layers x "
                               "{q,k,v,o,gate,up,down} + lm_head, distinct weights per layer, whole op "
                               "(row quant + product) per Linear; Linears that share an input (q,k,v; "
                               "gate,up) are issued as one grouped call"
                               + (f"; down_proj's k range is dealt to {kparts} workgroups per tile row and its "
                                  "partial rows are added up by the launch that reads them (the next layer's "
                                  "q,k,v)" if split_down else ""),
                   "M": 1, "linears": len(step_linears), "launches": n_launch,
                   "algorithmic_bytes_per_step": step_bytes},
        "roofline": roofline, "cpu_baseline": cpu,
        # the other two figures the headline metric names, measured in the same run (details in extra)
        "also": {"prefill_gemm_TFLOPs_M512_gate_proj": (extra.get("prefill_roofline") or {}).get(
                     "M512_gate_proj_kernel_TFLOPs"),
                 "prefill_layer_TFLOPs_M512_as_issued": ((extra.get("prefill") or {}).get("M512") or {}).get(
                     "layer_as_issued_TFLOPs"),
                 "decoder_tokens_per_s_batch1": (extra.get("decoder_config4") or {}).get("decode_tokens_per_s"),
                 "decoder_prefill_tokens_per_s_512": (extra.get("decoder_config4") or {}).get(
                     "prefill_tokens_per_s")},
        "extra": extra,
    }
    print(json.dumps(out))


if __name__ == "__main__":
    main()
