"""CPU: the layered decoder's oracle pinned by closed forms and torch's own operators, and the parts of the product that need
no GPU (configuration checks, sizes, the programs' usage)."""
import ctypes
import os
import subprocess

import numpy as np
import pytest
import torch

import layered_models as lm
import layered_oracle as lo

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
rng = np.random.default_rng(3)


def test_norms_convolution_and_polynorm_against_torch():
    x = rng.standard_normal((7, 20)) * 3 + 1
    w = rng.standard_normal(20)
    t = torch.nn.functional.layer_norm(torch.tensor(x), (20,), torch.tensor(w), None, 1e-3).numpy()
    assert np.allclose(lo.layer_norm(x, w, 1e-3), t, atol=1e-12)
    k = rng.standard_normal((20, 4))
    pad = torch.nn.functional.pad(torch.tensor(x.T)[None], (3, 0))
    t = torch.nn.functional.conv1d(pad, torch.tensor(k)[:, None], groups=20)[0].numpy().T
    assert np.allclose(lo.causal_conv(x, k), t, atol=1e-12)
    assert np.allclose(lo.causal_conv(x, k[:, :1]), x * k[:, 0])
    rms = lambda z: z / np.sqrt((z * z).mean(-1, keepdims=True) + 1e-5)
    assert np.allclose(lo.polynorm(x, (2.0, 0, 0, 0.5), 1e-5), 2 * rms(x) + 0.5)
    assert np.allclose(lo.polynorm(x, (0, -1.0, 3.0, 0), 1e-5), 3 * rms(x ** 3) - rms(x * x))


def test_pooled_window_attention_against_plain_causal_attention_and_visible_sets():
    T, H, G, d, dv = 23, 4, 2, 8, 6
    q, k, v = rng.standard_normal((T, H, d)), rng.standard_normal((T, G, d)), rng.standard_normal((T, G, dv))
    ref = torch.nn.functional.scaled_dot_product_attention(
        torch.tensor(q).transpose(0, 1), torch.tensor(np.repeat(k, 2, 1)).transpose(0, 1),
        torch.tensor(np.repeat(v, 2, 1)).transpose(0, 1), is_causal=True, scale=0.3).transpose(0, 1).numpy()
    assert np.allclose(lo.pooled_window_attention(q, k, v, 0.3, T, 5), ref)
    # equal scores: the mean over what is visible, blocks counted once each
    for size, pool in [(1, 1), (4, 3), (5, 2), (3, 7)]:
        out = lo.pooled_window_attention(q, k, v, 0.0, size, pool)
        for i in range(T):
            seen = [v[j] for j in range(T) if 0 <= i - j < size]
            seen += [v[b * pool:(b + 1) * pool].mean(0) for b in range(T) if (b + 1) * pool - 1 <= i - size]
            assert np.allclose(out[i], np.repeat(np.mean(seen, 0), 2, 0))


def test_delta_rule_overwrites_and_retention_sums():
    d, dv = 6, 4
    e = np.eye(d)
    v = rng.standard_normal((5, 1, dv))
    one = np.ones((5, 1))
    keys = e[[0, 1, 0, 2, 1]][:, None]
    q = e[[0, 1, 0, 1, 1]][:, None]
    out = lo.delta_rule(q, keys, v, one, one)           # beta 1, no decay: an associative memory
    assert np.allclose(out[:, 0], v[[0, 1, 2, 1, 4], 0])
    half = lo.delta_rule(q, keys, v, one * 0.5, one)    # decays by 0.5 per token, overwriting is still exact
    assert np.allclose(half[3, 0], 0.25 * v[1, 0]) and np.allclose(half[4, 0], v[4, 0])
    assert np.allclose(lo.delta_rule(q, keys, v, one, 0 * one), 0)
    q, k = rng.standard_normal((2, 5, 1, d))
    out = lo.retention(q, k, v, [0.7])
    for t in range(5):
        want = sum(0.7 ** (t - s) * (q[t, 0] @ k[s, 0]) * v[s, 0] for s in range(t + 1))
        assert np.allclose(out[t, 0], want)


def test_rotation_is_relative_and_leaves_the_rest():
    x, y = rng.standard_normal((2, 10))
    a = lo.rotate_half(x, 9, 6, 100.0) @ lo.rotate_half(y, 4, 6, 100.0)
    b = lo.rotate_half(x, 25, 6, 100.0) @ lo.rotate_half(y, 20, 6, 100.0)
    assert np.isclose(a, b)
    assert np.array_equal(lo.rotate_half(x, 9, 6, 100.0)[6:], x[6:])
    u, v = x[0], x[3]                                    # the first pair turns by the position itself
    assert np.allclose(lo.rotate_half(x, 2, 6, 100.0)[[0, 3]],
                       [u * np.cos(2) - v * np.sin(2), v * np.cos(2) + u * np.sin(2)])


def test_sink_attention_against_torch_with_one_more_key():
    """A sink is a key whose score is the sink and whose value is zero."""
    T, H, G, d, dv = 17, 4, 2, 8, 6
    q, k, v = rng.standard_normal((T, H, d)), rng.standard_normal((T, G, d)), rng.standard_normal((T, G, dv))
    sinks = rng.standard_normal(H) * 2
    for size in (None, 1, 5, 40):
        i, j = np.arange(T)[:, None], np.arange(T)[None]
        mask = np.where((j <= i) & (i - j < (size or T)), 0.0, -np.inf)
        mask = np.concatenate([np.repeat(mask[None], H, 0), np.repeat(sinks[:, None, None], T, 1)], 2)
        more = lambda x: torch.tensor(np.concatenate([np.repeat(x, 2, 1).transpose(1, 0, 2), np.zeros((H, 1, x.shape[2]))], 1))
        ref = torch.nn.functional.scaled_dot_product_attention(torch.tensor(q.transpose(1, 0, 2)), more(k), more(v),
                                                               attn_mask=torch.tensor(mask), scale=0.4).numpy()
        assert np.allclose(lo.sink_attention(q, k, v, 0.4, sinks, size), ref.transpose(1, 0, 2))


def test_latent_attention_reads_what_its_folded_form_reads():
    """Scores and values taken in the latent space: query times W_uk, output times W_uv."""
    cfg = lm.lesarax([lm.latent(3, 6, 4, 5, 9, 7, 4)], width=12)
    w, m = lm.lesarax_weights(cfg, seed=2), cfg["layers"][0]["mixer"]
    p, T, H = "l0.mix.", 11, 3
    h = rng.standard_normal((T, 12))
    q = (lo.rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], 1e-5) @ w[p + "uq"].T).reshape(T, H, 10)
    ckv = h @ w[p + "dkv"].T
    c, uk, uv = lo.rms_norm(ckv[:, :7], w[p + "dkv.norm"], 1e-5), w[p + "uk"].reshape(3, 6, 7), w[p + "uv"].reshape(3, 5, 7)
    out = np.zeros((T, H, 5))
    for t in range(T):
        seen = range(max(0, t - 3), t + 1)
        for i in range(H):
            qr = lo.rotate_half(q[t, i, 6:], t, 4, 3000.0)
            s = [(uk[i].T @ q[t, i, :6]) @ c[j] + qr @ lo.rotate_half(ckv[j, 7:], j, 4, 3000.0) for j in seen]
            e = np.exp(np.array(s) * m["scale"])
            out[t, i] = uv[i] @ (e @ c[list(seen)]) / (e.sum() + np.exp(w[p + "sink"][i]))
            out[t, i] *= lo.sigmoid(w[p + "g"] @ h[t])[i]
    assert np.allclose(lo.mixer_latent_attention(cfg, w, p, m, h), out.reshape(T, -1) @ w[p + "o"].T)


def test_experts_norm_and_layer_runs():
    x = rng.standard_normal((4, 9))
    assert np.allclose(lo.rms_norm(x, np.ones(9), 0.0), torch.nn.functional.rms_norm(torch.tensor(x), (9,)).numpy())
    pick, a = lo.route(np.array([0.1, 3.0, -2.0, 2.0]), 2)
    assert list(pick) == [1, 3] and np.allclose(a, [1 / (1 + np.exp(-1)), 1 / (1 + np.exp(1))])
    one, zero = np.eye(3), np.zeros((3, 3))
    h = np.array([0.5, -0.7, 4.0])
    g = np.minimum(h, 1.5)
    assert np.allclose(lo.clamped_expert(h, one, zero, one, 1.5), g * lo.sigmoid(1.702 * g))
    assert np.allclose(lo.clamped_expert(h, one, one, 2 * one, 1.5), 2 * g * lo.sigmoid(1.702 * g) * (np.clip(h, -1.5, 1.5) + 1))
    assert np.allclose(lo.clamped_expert(-h, one, one, one, 1.5)[2], -4 * lo.sigmoid(1.702 * -4.0) * -0.5)   # g has no lower limit
    layers = [lm.rotary(1, 1, 8, 4)] * 4
    assert lo.layer_runs(lm.lesarax(layers, loop=(1, 3, 2))) == [(0, 0), (1, 1), (2, 0), (1, 1), (2, 0), (3, 0)]
    assert lo.layer_runs(lm.lesarax(layers, loop=(0, 1, 3))) == [(0, 1), (0, 1), (0, 1), (1, 0), (2, 0), (3, 0)]


def test_safetensors_round_trip(tmp_path):
    w = {"a.b": lo.bf16_round(rng.standard_normal((3, 5))), "c": lo.bf16_round(rng.standard_normal(7) * 1e-3)}
    lo.save_safetensors(tmp_path / "m", w)
    back = lo.load_safetensors(tmp_path / "m")
    assert set(back) == set(w) and all(np.array_equal(back[k], w[k]) for k in w)


def _cfg(pkg, cfg, dtype=1, max_seq=64, batch=16):
    """The C structure of a configuration, without weights."""
    arr = (pkg.LayerConfig * len(cfg["layers"]))()
    for c, layer in zip(arr, cfg["layers"]):
        m = layer["mixer"]
        c.mixer, c.heads, c.kv_heads = pkg.MIXERS[layer["type"]], m["heads"], m.get("kv_heads", m["heads"])
        c.dim, c.vdim, c.conv_taps, c.kv_from = m["dim"], m["vdim"], m.get("conv", 0), m.get("kv_from", -1)
        if layer["type"] == "attention":
            c.scale, c.window, c.pool = m["scale"], m["mask"]["size"], m["mask"]["pool"]
        if layer["type"] == "retention":
            c.rot_dims, c.rot_base = m["rot"]["dims"], m["rot"]["base"]
        c.ff = layer["mlp"]["ff"] if layer["mlp"] else 0
    return pkg.LayeredConfig(cfg["width"], cfg["vocab"], len(arr), cfg["canon"]["taps"], cfg["norm"]["eps"], dtype, max_seq,
                             batch, arr), arr


def test_configurations_that_cannot_run_are_refused(pkg):
    L = pkg.lib()
    A, D, R = lm.attention(2, 1, 16, 16, 5, 2), lm.delta(2, 1, 16, 8), lm.retention(2, 16, 8, 8)

    def code(layers, change=None, **kw):
        cfg, arr = _cfg(pkg, lm.config(layers, **kw))
        if change:
            change(cfg, arr)
        rc = L.w4a32_layered_check(ctypes.byref(cfg))
        assert (rc == 0) == (L.w4a32_layered_state_bytes(ctypes.byref(cfg)) > 0)
        assert (rc == 0) == (L.w4a32_layered_workspace_bytes(ctypes.byref(cfg)) > 0)
        return rc

    def field(i, name, value):
        return lambda cfg, arr: setattr(arr[i], name, value)

    EINVAL, ESHAPE, ENOTSUP = -1, -2, -4
    assert code([A, D, R, lm.attention(4, 1, 16, 16, 9, 3, kv_from=0)]) == 0
    assert code([A], field(0, "kv_heads", 3)) == ESHAPE
    assert code([A], field(0, "window", 0)) == EINVAL
    assert code([A], field(0, "pool", 0)) == EINVAL
    assert code([A], field(0, "dim", 300)) == ENOTSUP
    assert code([A], field(0, "conv_taps", 9)) == ENOTSUP
    assert code([A, lm.attention(2, 1, 16, 16, 5, 2, kv_from=1)]) == ESHAPE     # itself
    assert code([D, lm.attention(2, 1, 16, 16, 5, 2, kv_from=0)]) == ESHAPE     # not an attention layer
    assert code([A, lm.attention(2, 1, 24, 16, 5, 2, kv_from=0)]) == ESHAPE     # other sizes
    assert code([D], field(0, "conv_taps", 0)) == EINVAL
    assert code([R], field(0, "rot_dims", 7)) == ESHAPE
    assert code([R], field(0, "rot_dims", 18)) == ESHAPE
    assert code([R], field(0, "mixer", 9)) == EINVAL
    assert code([A], taps=0) == EINVAL and code([A], taps=9) == ENOTSUP
    assert code([A], lambda cfg, arr: setattr(cfg, "dtype", 3)) == EINVAL


def test_rotary_latent_experts_and_loops_are_checked(pkg):
    L = pkg.lib()

    def cfg_of(change=None, experts=4, loop=(0, 1, 2)):
        arr = (pkg.LayerConfig * 2)()
        a, b = arr
        a.mixer, a.heads, a.kv_heads, a.dim, a.vdim, a.kv_from = pkg.MIXERS["rotary"], 4, 2, 24, 24, -1
        a.tied_values, a.rot_dims, a.rot_base, a.scale = 1, 12, 1e4, 0.2
        b.mixer, b.heads, b.kv_heads, b.dim, b.vdim, b.kv_from = pkg.MIXERS["latent"], 3, 3, 24, 20, -1
        b.q_rank, b.kv_rank, b.rot_part, b.rot_dims, b.rot_base, b.scale, b.window = 30, 40, 8, 8, 1e4, 0.2, 5
        for c in arr:
            c.ff, c.experts, c.top, c.expert_limit = 32, experts, 2, 1.0
        cfg = pkg.LayeredConfig(48, 30, 2, 0, 1e-5, 1, 64, 16, arr, pkg.NORM_RMS, 0.5, *loop)
        if change:
            change(cfg, a, b)
        return cfg, arr

    def code(change=None, **kw):
        cfg, arr = cfg_of(change, **kw)
        return L.w4a32_layered_check(ctypes.byref(cfg))

    def set_(i, **kw):
        return lambda *c: [setattr(c[i], k, v) for k, v in kw.items()]

    EINVAL, ESHAPE, ENOTSUP = -1, -2, -4
    assert code() == 0
    assert code(set_(0, norm=pkg.NORM_LAYER)) == EINVAL        # layer norm comes with the input convolution
    assert code(set_(0, norm=7)) == EINVAL
    assert code(set_(0, loop_times=-1)) == EINVAL
    assert code(loop=(1, 3, 2)) == ESHAPE and code(loop=(1, 1, 2)) == ESHAPE and code(loop=(-1, 1, 2)) == ESHAPE
    assert code(loop=(0, 0, 0)) == 0
    assert code(set_(1, rot_dims=13)) == ESHAPE and code(set_(1, rot_dims=26)) == ESHAPE
    assert code(set_(1, vdim=20)) == ESHAPE                     # tied values are as long as the keys
    assert code(set_(1, vdim=20, tied_values=0)) == 0
    assert code(set_(1, conv_taps=3)) == ENOTSUP and code(set_(1, heads=66)) == ENOTSUP
    assert code(set_(1, rot_base=0.0)) == EINVAL and code(set_(1, window=-1)) == EINVAL
    assert code(set_(2, kv_heads=1)) == ESHAPE and code(set_(2, rot_dims=10)) == ESHAPE
    assert code(set_(2, q_rank=0)) == EINVAL and code(set_(2, kv_rank=0)) == EINVAL
    assert code(set_(2, kv_rank=513)) == ENOTSUP and code(set_(2, rot_part=130)) == ENOTSUP
    assert code(set_(2, window=0)) == 0 and code(set_(2, rot_part=0, rot_dims=0)) == 0
    assert code(set_(1, top=5)) == EINVAL and code(set_(1, top=0)) == EINVAL and code(set_(1, expert_limit=0.0)) == EINVAL
    assert code(experts=513) == ENOTSUP and code(set_(1, experts=64, top=17)) == ENOTSUP
    assert code(set_(1, ff=40000)) == ENOTSUP
    # a looped layer has a cache per pass; a latent layer keeps its latent and key part only
    runs = lambda **kw: (lambda c: (L.w4a32_layered_runs(ctypes.byref(c[0])), L.w4a32_layered_state_bytes(ctypes.byref(c[0]))))(
        cfg_of(**kw))
    (n1, one), (n3, three) = runs(loop=(0, 1, 1)), runs(loop=(0, 1, 3))
    assert (n1, n3) == (2, 4) and three - one == 2 * 2 * 2 * 2 * 64 * 32
    assert L.w4a32_layered_head_rows(24, 20) == 32 and L.w4a32_layered_head_rows(24, 130) == 256


def test_a_layer_that_reads_another_ones_keys_keeps_no_cache_of_its_own(pkg):
    L = pkg.lib()

    def state(layers):
        cfg, arr = _cfg(pkg, lm.config(layers), max_seq=4096)
        return L.w4a32_layered_state_bytes(ctypes.byref(cfg))

    own = lm.attention(2, 1, 64, 64, 9, 8)
    one, two = state([own]), state([own, own])
    shared = state([own, lm.attention(2, 1, 64, 64, 30, 8, kv_from=0)])
    other_pool = state([own, lm.attention(2, 1, 64, 64, 30, 4, kv_from=0)])
    cache = 2 * 2 * 4096 * 64                       # keys and values, bf16
    assert two - one > cache and shared - one < cache / 8
    assert shared < other_pool < two                # block means of another size are kept, keys are not


@pytest.mark.parametrize("program", ["trace_run", "generate"])
def test_programs_print_their_usage(program):
    out = subprocess.run([os.path.join(ROOT, "bin", program), "--model"], capture_output=True, text=True, timeout=900)
    assert out.returncode == 2 and "usage: " + program in out.stderr
