"""GPU: rotary attention with sinks and tied values, latent attention, mixtures of experts and looped layers on the layered
decoder, against its float64 oracle: operators, each mechanism alone, portions of prompts, decoding, window edges, keys far
back, the first tokens, states used again, greedy generation, and the two programs."""
import ctypes
import json
import os

import numpy as np
import pytest

import layered_models as lm
import layered_oracle as lo
from test_gpu_layered import DTYPES, TOL, _cli, cuts, run

pytestmark = pytest.mark.gpu

M = lm.moe(40, 5, 2)
MODELS = {
    "rotary": ([lm.rotary(4, 2, 40, 24)], (0, 1, 1)),
    "rotary one head, all of it rotated": ([lm.rotary(1, 1, 32, 32)], (0, 1, 1)),
    "rotary odd half": ([lm.rotary(6, 2, 20, 6)], (0, 1, 1)),
    "rotary wide heads": ([lm.rotary(2, 1, 200, 66)], (0, 1, 1)),
    "rotary many heads on one key": ([lm.rotary(32, 1, 16, 8)], (0, 1, 1)),
    "latent": ([lm.latent(4, 24, 8, 40, 28, 36, 33)], (0, 1, 1)),
    "latent window of one": ([lm.latent(2, 32, 16, 32, 64, 64, 1)], (0, 1, 1)),
    "latent window past the sequence": ([lm.latent(3, 13, 6, 11, 17, 23, 500)], (0, 1, 1)),
    "latent more heads than a block": ([lm.latent(35, 16, 16, 8, 40, 100, 64)], (0, 1, 1)),
    "latent wide": ([lm.latent(2, 130, 70, 200, 200, 300, 47)], (0, 1, 1)),
    "latent rank 512": ([lm.latent(2, 64, 32, 64, 96, 512, 70)], (0, 1, 1)),
    "experts": ([lm.rotary(1, 1, 16, 8, mlp=lm.moe(100, 7, 3))], (0, 1, 1)),
    "one expert": ([lm.rotary(1, 1, 16, 8, mlp=lm.moe(33, 1, 1, 0.4))], (0, 1, 1)),
    "all of many experts": ([lm.rotary(1, 1, 16, 8, mlp=lm.moe(16, 16, 16, 5.0))], (0, 1, 1)),
    "experts beyond a wavefront": ([lm.rotary(1, 1, 16, 8, mlp=lm.moe(8, 70, 1))], (0, 1, 1)),
    "loop of everything": ([lm.rotary(2, 1, 16, 8), lm.latent(2, 16, 8, 16, 24, 32, 9)], (0, 2, 3)),
    "loop in the middle": ([lm.latent(2, 16, 8, 16, 24, 32, 20, mlp=M), lm.rotary(2, 2, 24, 8), lm.rotary(4, 2, 16, 16, mlp=M),
                            lm.latent(3, 16, 4, 24, 24, 32, 13)], (1, 3, 2)),
    "all kinds": ([lm.rotary(4, 2, 40, 24, mlp=M), lm.latent(4, 24, 8, 40, 28, 36, 33, mlp=M), lm.latent(2, 40, 16, 16, 50, 70, 12),
                   lm.rotary(2, 1, 64, 10, mlp=lm.moe(70, 9, 4))], (1, 3, 2)),
}


def model(name, seed=None, dtype="float32", **kw):
    """bfloat16: several layers in a row choose all of their experts, since rounding in one layer turns close calls of the next
    ones (the choice itself is tested alone, in layers by themselves and in float32)."""
    layers, loop = json.loads(json.dumps(MODELS[name]))
    if dtype == "bfloat16" and len(layers) > 1:
        for layer in layers:
            if layer["mlp"]:
                layer["mlp"]["router"]["top"] = layer["mlp"]["router"]["experts"]
    cfg = lm.lesarax(layers, loop=loop, **kw)
    return cfg, lm.lesarax_weights(cfg, seed=len(name) if seed is None else seed)


# ---------------------------------------------------------------------------------------------- operators
@pytest.mark.parametrize("rows,hidden,experts,top,ff", [(1, 64, 3, 2, 20), (5, 100, 9, 4, 64), (130, 200, 6, 3, 100),
                                                        (700, 72, 5, 2, 130), (300, 64, 80, 1, 40), (40, 64, 512, 16, 8)])
def test_experts_alone(pkg, rows, hidden, experts, top, ff):
    """Every (token, slot) row against the expert of that slot; experts nobody or everybody chooses are among them."""
    import torch

    rng = np.random.default_rng(rows + experts)
    h = lo.bf16_round(rng.standard_normal((rows, hidden)))
    gate, up = (lo.bf16_round(rng.standard_normal((experts, ff, hidden)) * 1.5 * hidden ** -0.5) for _ in range(2))
    down = lo.bf16_round(rng.standard_normal((experts, hidden, ff)) * ff ** -0.5)
    logits = np.stack([rng.permutation(experts) * 0.3 for _ in range(rows)])     # no close calls
    logits[:, experts // 2] += 1000.0 if experts > 1 else 0.0
    logits = logits.astype(np.float32).astype(np.float64)
    pad = lambda n: (n + 63) // 64 * 64
    for dtype, tol in ((torch.float32, 3e-6), (torch.bfloat16, 1e-2)):
        dev = lambda a: torch.tensor(a, device="cuda").to(dtype)
        hp = torch.zeros((rows, pad(hidden)), dtype=dtype, device="cuda")
        hp[:, :hidden] = dev(h)
        dp = torch.zeros((experts, pad(hidden), pad(ff)), dtype=dtype, device="cuda")
        dp[:, :hidden, :ff] = dev(down)
        parts = pkg.op_experts(hp, torch.tensor(logits, dtype=torch.float32, device="cuda"), pkg.pack_gate_up(dev(gate), dev(up)),
                               dp, hidden, top, ff, 0.9).double().cpu().numpy()
        assert np.all(parts[:, :, hidden:] == 0)
        for t in rng.permutation(rows)[:25]:
            for slot, (e, a) in enumerate(zip(*lo.route(logits[t], top))):
                ref = a * lo.clamped_expert(h[t], gate[e], up[e], down[e], 0.9)
                assert np.abs(parts[slot, t, :hidden] - ref).max() < tol * (np.abs(ref).max() + 1e-9) + 1e-12, (t, slot)


def test_experts_with_logits_that_do_not_compare_stay_in_bounds(pkg):
    import torch

    w = torch.ones((3, 64, 64), device="cuda")
    logits = torch.full((70, 3), float("nan"), device="cuda")
    out = pkg.op_experts(torch.ones((70, 64), device="cuda"), logits, pkg.pack_gate_up(w, w), w, 64, 2, 64, 1.0)
    assert out.shape == (2, 70, 64)
    torch.cuda.synchronize()


@pytest.mark.parametrize("H,taps", [(100, 0), (330, 2), (2304, 0)])
def test_rms_norm_of_the_residual_stream(pkg, H, taps):
    """The norm kernels' plain form, through a model of one layer whose sublayers add nothing."""
    cfg = lm.lesarax([lm.rotary(1, 1, 16, 8, mlp=lm.moe(8, 2, 1))], width=H, mult=0.0 if taps == 0 else 1e-30, eps=1e-2)
    w = lm.lesarax_weights(cfg, seed=H)
    w["l0.mix.o"][:] = 0
    for e in range(2):
        w[f"l0.mlp.e{e}.down"][:] = 0
    tokens = np.random.default_rng(H).integers(0, cfg["vocab"], 9)
    ref = lo.forward(cfg, w, tokens)
    for portions in ([9], [1] * 9):
        dec = lm.runner(cfg, w, "float32", 12)
        assert lm.errors(run(dec, dec.new_state(), tokens, portions), ref).max() < TOL["float32"]


# ---------------------------------------------------------------------------------------------- mechanisms alone, together
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", MODELS)
def test_prefill_decoding_and_portions_agree_with_the_oracle(name, dtype):
    cfg, w = model(name, dtype=dtype)
    T = 110
    tokens = np.random.default_rng(1).integers(0, cfg["vocab"], T)
    ref = lo.forward(cfg, w, tokens)
    dec = lm.runner(cfg, w, dtype, T + 3)
    state = dec.new_state()
    # the one state serves every run: each starts at position 0 on what the last one left
    for portions in ([T], cuts(T, 64), cuts(T, 2), cuts(T, 17, 1, 3, 31, 2), [70] + [1] * 40, [1] * T):
        e = lm.errors(run(dec, state, tokens, portions), ref)
        # (a close call between experts that bf16 rounding turned: few positions of one layer's choice)
        assert np.median(e) < TOL[dtype] / 2 and np.mean(e > TOL[dtype]) <= (0.0 if dtype == "float32" else 0.03), \
            (portions[:4], e.max(), int(e.argmax()))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,vocab,mult,eps", [(64, 40, 1.0, 1e-5), (200, 301, 0.25, 1e-3), (2500, 64, 1.5, 1e-6)])
def test_other_sizes(width, vocab, mult, eps, dtype):
    cfg = lm.lesarax([lm.latent(3, 20, 10, 28, 45, 50, 21), lm.rotary(3, 3, 28, 14, mlp=lm.moe(50, 4, 4, 0.7))], width, vocab,
                     (1, 2, 2), mult, eps)
    w = lm.lesarax_weights(cfg, seed=width)
    tokens = np.random.default_rng(2).integers(0, vocab, 70)
    ref = lo.forward(cfg, w, tokens)
    dec = lm.runner(cfg, w, dtype, 80)
    for portions in ([70], cuts(70, 9, 2), [1] * 70):
        e = lm.errors(run(dec, dec.new_state(), tokens, portions), ref)
        assert e.max() < TOL[dtype], (portions[:3], e.max())


def test_residual_stream_behind_every_layer_run(pkg):
    cfg, w = model("all kinds")
    tokens = np.random.default_rng(3).integers(0, cfg["vocab"], 30)
    layers = []
    lo.forward(cfg, w, tokens, layers)
    dec = lm.runner(cfg, w, "float32", 40)
    assert pkg.lib().w4a32_layered_runs(ctypes.byref(dec.cfg)) == len(layers) == 6
    for n, want in enumerate(layers, 1):
        got = dec.residual(dec.new_state(), tokens, 0, n).double().cpu().numpy()
        assert np.abs(got - want).max() < 2e-5 * np.abs(want).max()
        state = dec.new_state()
        dec.residual(state, tokens[:-1], 0, n)
        last = dec.residual(state, tokens[-1:], 29, n).double().cpu().numpy()
        assert np.abs(last[0] - want[-1]).max() < 2e-5 * np.abs(want).max()


# ---------------------------------------------------------------------------------------------- what must show
KEY, QUERY, FILL = 20, 21, 20    # tokens 0 .. 19 fill, QUERY asks for KEY


def spotlight(cfg, w, layer=0, gain=7.0):
    """One pair of tokens stands out: KEY's key and QUERY's query point the same way in every head of a layer."""
    m, p = cfg["layers"][layer]["mixer"], f"l{layer}.mix."
    rng = np.random.default_rng(9)
    W, H = cfg["width"], m["heads"]
    w[f"l{layer}.norm1"][:] = 1
    w["loop.in"] = np.concatenate([np.eye(W), np.zeros((W, W))], 1)
    emb = w["embed"]
    basis = np.linalg.qr(np.stack([emb[KEY], emb[QUERY]]).T)[0]
    rest = [t for t in range(cfg["vocab"]) if t not in (KEY, QUERY)]
    emb[rest] -= emb[rest] @ basis @ basis.T
    emb[KEY], emb[QUERY] = basis[:, 0] * W ** 0.5, basis[:, 1] * W ** 0.5
    at = {t: emb[t] / W for t in (KEY, QUERY)}          # picks the token's share out of a normed row
    one = lambda n: (lambda v: v / np.linalg.norm(v))(rng.standard_normal(n))
    if cfg["layers"][layer]["type"] == "attention":
        free = m["dim"] - m["rot"]["dims"]                 # the unrotated dimensions do not depend on the distance
        dirs = np.stack([np.concatenate([np.zeros(m["rot"]["dims"]), one(free)]) for _ in range(m["kv_heads"])])
        rep = H // m["kv_heads"]
        w[p + "q"] = w[p + "q"] * 0.2 + gain * np.repeat(dirs, rep, 0).reshape(-1)[:, None] * at[QUERY]
        w[p + "k"] = w[p + "k"] * 0.2 + gain * dirs.reshape(-1)[:, None] * at[KEY]
    else:
        uq, uc = one(m["q_rank"]), one(m["kv_rank"])
        dirs = np.stack([one(m["dim"]) for _ in range(H)])
        w[p + "dq"] += 4 * m["q_rank"] ** 0.5 * uq[:, None] * at[QUERY]
        w[p + "dkv"][:m["kv_rank"]] += 4 * m["kv_rank"] ** 0.5 * uc[:, None] * at[KEY]
        up = np.concatenate([dirs, np.zeros((H, m["rot_dim"]))], 1).reshape(-1)
        w[p + "uq"] = w[p + "uq"] * 0.2 + gain * m["q_rank"] ** -0.5 * up[:, None] * uq
        w[p + "uk"] = w[p + "uk"] * 0.2 + gain * m["kv_rank"] ** -0.5 * dirs.reshape(-1)[:, None] * uc
    w[p + "sink"][:] = 2.0
    w[p + "o"] *= 3
    for name in w:
        w[name] = lo.bf16_round(w[name])


def planted(monkeypatch, cfg, w, tokens, **functions):
    """The oracle's logits with other functions in it."""
    with monkeypatch.context() as mp:
        for name, f in functions.items():
            mp.setattr(lo, name, f)
        return lo.forward(cfg, w, tokens)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size", [1, 2, 9, 31, 32, 33, 64, 70])
def test_keys_just_inside_and_outside_of_the_window(monkeypatch, size, dtype):
    cfg = lm.lesarax([lm.latent(4, 24, 8, 40, 28, 36, size)], mult=1.0)
    w = lm.lesarax_weights(cfg, seed=size)
    spotlight(cfg, w)
    plain = lo.sink_attention
    moved = lambda by: lambda q, k, v, scale, sinks, n: plain(q, k, v, scale, sinks, n + by)
    rng = np.random.default_rng(size)
    dec = lm.runner(cfg, w, dtype, 160)
    state = dec.new_state()
    for name, key_at, query_at, wrong in (("in", 40, 40 + size - 1, moved(-1)), ("out", 40, 40 + size, moved(1)),
                                          ("first token in", 0, size - 1, moved(-1)), ("first token out", 0, size, moved(1)),
                                          ("edge of a block", 31, 31 + size, moved(1))):
        if key_at == query_at:
            continue
        tokens = rng.integers(0, FILL, query_at + 1)
        tokens[key_at], tokens[query_at] = KEY, QUERY
        ref, bad = lo.forward(cfg, w, tokens), planted(monkeypatch, cfg, w, tokens, sink_attention=wrong)
        shows = lm.errors(bad, ref)[query_at]
        n = len(tokens)
        for portions in ([n], [n - 1, 1], cuts(n, 13), cuts(n, 2), cuts(n, max(1, n - 3), 2, 1)):
            e = lm.errors(run(dec, state, tokens, portions), ref)[query_at]
            assert e < TOL[dtype] * (1 if dtype == "float32" else 2) and shows > max(10 * e, 0.05), (name, portions, e, shows)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_key_far_back(monkeypatch, dtype):
    """Rotary attention sees every token: one 300 tokens back, in a prompt, behind portions and in decoding."""
    cfg = lm.lesarax([lm.rotary(4, 2, 40, 16)], mult=1.0)
    w = lm.lesarax_weights(cfg, seed=4)
    spotlight(cfg, w)
    plain = lo.sink_attention
    T = 330
    dec = lm.runner(cfg, w, dtype, 340)
    for key_at in (0, 1, 31, 32, 27):
        tokens = np.random.default_rng(6).integers(0, FILL, T)
        tokens[key_at], tokens[-1] = KEY, QUERY
        ref = lo.forward(cfg, w, tokens)
        bad = planted(monkeypatch, cfg, w, tokens, sink_attention=lambda q, k, v, s, z, n=None: plain(q, k, v, s, z, T - key_at - 1))
        shows = lm.errors(bad, ref)[-1]
        for portions in ([T], cuts(T, 64), cuts(T, 2), [5] + [1] * (T - 5), [T - 1, 1]):
            e = lm.errors(run(dec, dec.new_state(), tokens, portions), ref)[-1]
            assert e < TOL[dtype] and shows > max(10 * e, 0.05), (key_at, portions[:3], e, shows)


MISTAKES = {
    "sinks left out": ("all kinds", {"sink_attention": lambda f: lambda q, k, v, s, z, n=None: f(q, k, v, s, z - 1e9, n)}),
    "sinks scaled": ("all kinds", {"sink_attention": lambda f: lambda q, k, v, s, z, n=None: f(q, k, v, s, z * s, n)}),
    "rotated keys as values": ("rotary", {"sink_attention": lambda f: lambda q, k, v, s, z, n=None: f(q, k, k, s, z, n)}),
    "another base of the rotation": ("all kinds", {"rotate_half": lambda f: lambda x, p, d, b: f(x, p, d, b * 1.3)}),
    "gates left out": ("latent", {"sigmoid": lambda f: lambda x: np.ones_like(x)}),
    "limit left out": ("experts", {"clamped_expert": lambda f: lambda h, g, u, d, lim: f(h, g, u, d, 1e9)}),
    "softmax over all experts": ("experts", {"route": lambda f: lambda z, t: (f(z, t)[0], f(z, len(z))[1][:t])}),
    "one pass too few": ("loop of everything", {"layer_runs": lambda f: lambda c: f(c)[:-2]}),
    "input product of the first pass only": ("loop in the middle", {"layer_runs": lambda f: lambda c: [
        (i, s and f(c).index((i, s)) == k) for k, (i, s) in enumerate(f(c))]}),
    "mean taken off in the norm": ("all kinds", {"rms_norm": lambda f: lambda x, w, e: f(x - x.mean(-1, keepdims=True), w, e)}),
}


@pytest.mark.parametrize("mistake", MISTAKES)
def test_a_mistake_would_show(monkeypatch, mistake):
    """The mistake, planted in the oracle, is far outside of what separates the framework from the right one."""
    name, change = MISTAKES[mistake]
    cfg, w = model(name)
    tokens = np.random.default_rng(8).integers(0, cfg["vocab"], 60)
    ref = lo.forward(cfg, w, tokens)
    bad = planted(monkeypatch, cfg, w, tokens, **{k: f(getattr(lo, k)) for k, f in change.items()})
    dec = lm.runner(cfg, w, "float32", 64)
    for portions in ([60], [30] + [1] * 30):
        got = run(dec, dec.new_state(), tokens, portions)
        assert lm.errors(got, ref).max() < TOL["float32"] and np.median(lm.errors(got, bad)) > 30 * TOL["float32"]


def test_passes_of_a_loop_keep_caches_of_their_own(monkeypatch):
    """A key only one pass writes: both passes of the loop see their own, in portions and in decoding."""
    cfg, w = model("loop of everything")
    one = json.loads(json.dumps(cfg))
    one["loop"]["times"] = 1
    tokens = np.random.default_rng(10).integers(0, cfg["vocab"], 40)
    sizes = []
    for c in (one, cfg):
        dec = lm.runner(c, w, "float32", 2048, 64)
        sizes.append(dec.new_state().numel())
        ref = lo.forward(c, w, tokens)
        for portions in ([40], cuts(40, 3), [2] + [1] * 38):
            assert lm.errors(run(dec, dec.new_state(), tokens, portions), ref).max() < TOL["float32"]
    assert sizes[1] > 2.9 * sizes[0]


def test_first_tokens():
    cfg, w = model("all kinds")
    dec = lm.runner(cfg, w, "float32", 40)
    state = dec.new_state()
    run(dec, state, np.arange(40) % cfg["vocab"], [40])        # leaves full caches
    for tokens in ([7], [7, 3], [1, 2, 3], [5, 5, 5, 5, 5]):
        ref = lo.forward(cfg, w, tokens)
        for portions in ([len(tokens)], [1] * len(tokens)):
            assert lm.errors(run(dec, state, np.array(tokens), portions), ref).max() < TOL["float32"]


@pytest.mark.parametrize("dtype", DTYPES)
def test_sequences_do_not_see_each_other(dtype):
    """Several sequences through one workspace, a portion of each in turn; ended states serve new sequences."""
    cfg, w = model("loop in the middle", dtype=dtype)
    dec = lm.runner(cfg, w, dtype, 128)
    rng = np.random.default_rng(12)
    states = [dec.new_state() for _ in range(3)]
    for lengths in ([90, 17, 2], [3, 128, 60]):
        seqs = [rng.integers(0, cfg["vocab"], n) for n in lengths]
        refs = [lo.forward(cfg, w, s) for s in seqs]
        at, errs = [0, 0, 0], []
        while any(a < len(s) for a, s in zip(at, seqs)):
            for i, s in enumerate(seqs):
                n = min(len(s) - at[i], int(rng.choice([1, 2, 5, 33])))
                if n > 0:
                    got = dec.forward(states[i], s[at[i]:at[i] + n], at[i])
                    errs += list(lm.errors(got, refs[i][at[i]:at[i] + n]))
                    at[i] += n
        assert max(errs) < TOL[dtype]


def test_stale_memory_is_not_read():
    """A state whose cache rows past the sequence hold Inf and NaN gives the same logits."""
    import torch

    cfg = lm.lesarax([lm.rotary(4, 2, 40, 24), lm.latent(4, 24, 8, 40, 28, 36, 20), lm.rotary(2, 1, 16, 8)], loop=(1, 3, 2))
    w = lm.lesarax_weights(cfg, seed=15)
    tokens = np.random.default_rng(16).integers(0, cfg["vocab"], 75)
    for dtype in DTYPES:
        dec = lm.runner(cfg, w, dtype, 128)
        clean = run(dec, dec.new_state(), tokens, [50, 3] + [1] * 22)
        bad = lm.runner(cfg, {**w, "embed": np.full_like(w["embed"], np.inf)}, dtype, 128)
        state = bad.new_state()
        bad.forward(state, np.zeros(128, dtype=np.int64), 0, want=[])
        got = run(dec, state, tokens, [50, 3] + [1] * 22)
        assert torch.equal(got, clean)


def test_logits_do_not_depend_on_the_cut_beyond_rounding():
    """Wanted rows of a portion only, none, or all; large portions against small ones on a longer sequence."""
    cfg, w = model("all kinds", seed=13)
    T = 700
    tokens = np.random.default_rng(14).integers(0, cfg["vocab"], T)
    dec = lm.runner(cfg, w, "float32", T, 700)
    whole = dec.forward(dec.new_state(), tokens, 0).double().cpu().numpy()
    state = dec.new_state()
    at = 0
    for n in cuts(T, 200, 3, 64, 1, 2, 77):
        want = [k for k in range(n) if (at + k) % 7 == 0]
        got = dec.forward(state, tokens[at:at + n], at, want)
        if want:
            assert lm.errors(got, whole[at + np.array(want)]).max() < TOL["float32"]
        at += n


# ---------------------------------------------------------------------------------------------- decoding loop, programs
@pytest.mark.parametrize("dtype", DTYPES)
def test_long_greedy_decoding_from_a_graph(dtype):
    """Greedy steps replayed from a HIP graph, eager work in between, against the oracle fed with the chosen tokens."""
    import torch

    cfg, w = model("all kinds", seed=17, dtype=dtype)
    n_prompt, n_new = 21, 120
    prompt = np.random.default_rng(18).integers(0, cfg["vocab"], n_prompt)
    dec = lm.runner(cfg, w, dtype, 160)
    state, other = dec.new_state(), dec.new_state()
    stream = torch.cuda.Stream()
    with torch.cuda.stream(stream):
        dec.prefill(state, torch.tensor(prompt, device="cuda"))
        tokens = [int(dec.token)]
        dec.step(state)
        tokens.append(int(dec.token))
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph, stream=stream):
            dec.step(state)
        for i in range(n_new):
            if i % 29 == 0:                                   # other work in the same workspace
                keep = dec.token.clone()
                dec.forward(other, prompt[:1 + i % 4], 0)
                dec.token.copy_(keep)
            graph.replay()
            tokens.append(int(dec.token))
    fed = list(prompt) + tokens[:-1]
    ref = lo.forward(cfg, w, fed)[n_prompt - 1:]
    gaps = np.array([(ref[i].max() - ref[i][t]) / ref.std() for i, t in enumerate(tokens)])
    assert gaps.max() <= 6 * TOL[dtype]                       # the oracle's choice, or one rounding cannot tell from it
    assert np.mean(gaps == 0) > (0.99 if dtype == "float32" else 0.8)


@pytest.mark.parametrize("dtype", DTYPES)
def test_generate_program(tmp_path, dtype):
    """A model folder through the registry: three prompts one after the other (states used again, graph replay), in one
    slice and in slices of five tokens."""
    cfg, w = model("all kinds", seed=19, dtype=dtype)
    lm.write_model(tmp_path, cfg, w)
    rng = np.random.default_rng(20)
    prompts = [list(map(int, rng.integers(0, cfg["vocab"], n))) for n in (12, 1, 40)]
    args = [a for p in prompts for a in ("--tokens", ",".join(map(str, p)))]
    outs = []
    for chunk in ("64", "5"):
        out = _cli("generate", "--model", str(tmp_path), "--dtype", dtype, "--max-new", "25", "--max-tokens", "80",
                   "--chunk", chunk, *args)
        assert out.returncode == 0, out.stderr[-2000:]
        outs.append([list(map(int, line.split())) for line in out.stdout.strip().splitlines()])
    for gens in outs:
        assert [len(g) for g in gens] == [25, 25, 25]
        for p, g in zip(prompts, gens):
            ref = lo.forward(cfg, w, p + g[:-1])[len(p) - 1:]
            gaps = np.array([(ref[i].max() - ref[i][t]) / ref.std() for i, t in enumerate(g)])
            assert gaps.max() <= 6 * TOL[dtype]
    if dtype == "float32":
        assert outs[0] == outs[1]


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_run_program(tmp_path, dtype):
    cfg, w = model("loop in the middle", seed=21, dtype=dtype, vocab=61)
    lm.write_model(tmp_path / "model", cfg, w)
    os.mkdir(tmp_path / "out")
    rng = np.random.default_rng(22)
    lines, wanted, refs = [], [], {}
    for k, n in (("a", 70), ("b", 1), ("c", 33), ("d", 64)):
        seq = rng.integers(0, 61, n)
        refs[k] = lo.forward(cfg, w, seq)
        at = 0
        while at < n:
            m = min(n - at, int(rng.choice([1, 2, 3, 16, 40])))
            want = sorted(set(map(int, rng.integers(0, m, 2)))) if rng.random() < 0.8 else []
            wanted.append((k, [at + x for x in want]))
            lines.append(json.dumps({"step": len(lines), "end": [k] if at + m == n else [],
                                     "entries": [{"id": k, "tokens": list(map(int, seq[at:at + m])), "want": want}]}))
            at += m
    out = _cli("trace_run", "--model", str(tmp_path / "model"), "--dtype", dtype, "--out", str(tmp_path / "out"), "--max-tokens",
               "100", stdin="\n".join(lines) + "\n")
    assert out.returncode == 0, out.stderr[-2000:]
    assert [ln for ln in out.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(len(lines))]
    errs = []
    for i, (k, places) in enumerate(wanted):
        path = tmp_path / "out" / f"{i}.f32"
        if not places:
            assert not path.exists()
            continue
        got = np.fromfile(path, "<f4").reshape(len(places), 61).astype(np.float64)
        errs += list(lm.errors(got, refs[k][places]))
    assert max(errs) < TOL[dtype]


def test_the_file_s_weights_are_packed_as_the_binding_packs_them(tmp_path):
    """C++ loader and Python plumbing give the same logits to the last bit."""
    cfg, w = model("all kinds", seed=23)
    lm.write_model(tmp_path / "model", cfg, w)
    os.mkdir(tmp_path / "out")
    tokens = list(map(int, np.random.default_rng(24).integers(0, cfg["vocab"], 50)))
    line = json.dumps({"step": 0, "entries": [{"id": "a", "tokens": tokens, "want": list(range(50))}], "end": ["a"]})
    for dtype in DTYPES:
        out = _cli("trace_run", "--model", str(tmp_path / "model"), "--dtype", dtype, "--out", str(tmp_path / "out"),
                   "--max-tokens", "64", stdin=line + "\n")
        assert out.returncode == 0, out.stderr[-2000:]
        dec = lm.runner(cfg, w, dtype, 64)
        want = dec.forward(dec.new_state(), tokens, 0).cpu().numpy()
        assert np.array_equal(np.fromfile(tmp_path / "out" / "0.f32", "<f4").reshape(want.shape), want)


def test_programs_refuse_what_they_cannot_run(tmp_path):
    cfg = lm.lesarax([lm.latent(2, 16, 8, 16, 24, 32, 9, mlp=lm.moe(8, 3, 2))])
    w = lm.lesarax_weights(cfg)

    def stderr_of(change_cfg=None, change_w=None):
        c, ww = json.loads(json.dumps(cfg)), dict(w)
        if change_cfg:
            change_cfg(c)
        if change_w:
            change_w(ww)
        lm.write_model(tmp_path, c, ww)
        out = _cli("generate", "--model", str(tmp_path), "--max-tokens", "20", "--tokens", "1,2")
        assert out.returncode not in (0, -6, -11), out.stderr
        return out.stderr

    mixer = lambda **kw: lambda c: c["layers"][0]["mixer"].update(**kw)
    assert "mixer" in stderr_of(lambda c: c["layers"][0].update(type="unheard"))
    assert "feed-forward" in stderr_of(lambda c: c["layers"][0]["mlp"].update(kind="dense"))
    assert "cannot run" in stderr_of(lambda c: c["layers"][0]["mlp"]["router"].update(top=4))
    assert "cannot run" in stderr_of(mixer(kv_rank=600))
    assert "cannot run" in stderr_of(lambda c: c["loop"].update(stop=2))
    assert "shape" in stderr_of(mixer(q_rank=25))
    assert "l0.mlp.e2.down not found" in stderr_of(None, lambda ww: ww.pop("l0.mlp.e2.down"))
    assert "l0.mix.sink not found" in stderr_of(None, lambda ww: ww.pop("l0.mix.sink"))
