"""Bamudra against the plain float64 oracle in ``bamudra_oracle.py``.

Every test builds its own small configuration and random weights, runs the framework (config
reader, weight conversion, engine, scheduler, block manager, state slots, runner, model, ops)
and compares with the oracle's whole-sequence functions. CPU cases run the PyTorch reference
ops in fp32; GPU cases run the HIP kernels in bf16 and fp32.
"""
import copy

import numpy as np
import pytest
import torch

import bamudra_oracle as O
from distributed_llm_inferencing_amd.engine import SamplingParams
from distributed_llm_inferencing_amd.engine.llm_engine import LLMEngine
from distributed_llm_inferencing_amd.models.hf import config_from_hf
from distributed_llm_inferencing_amd.models.weights import from_bamudra_state_dict
from distributed_llm_inferencing_amd.ops import hybrid as H

CASES = [("cpu", torch.float32),
         pytest.param("cuda", torch.float32, marks=pytest.mark.gpu),
         pytest.param("cuda", torch.bfloat16, marks=pytest.mark.gpu)]


def dense(ff=40, limit=0.9):
    return {"kind": "dense", "ff": ff, "limit": limit}


def rot(dims=4, base=60.0):
    return {"base": base, "dims": dims}


def retention(heads=2, dim=8, vdim=12, decay=None, rot_=None, mlp=None):
    decay = decay or [1.0 - 0.4 * (i + 1) / (heads * (i + 2)) for i in range(heads)]
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay,
                                           "rot": rot() if rot_ is None else rot_}, "mlp": mlp}


def attention(heads=4, kv_heads=2, dim=8, scale=0.45, rot_=None, size=11, keep=3, mlp=None):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale,
                      "rot": rot(6) if rot_ is None else rot_,
                      "mask": {"size": size, "keep_first": keep}}, "mlp": mlp}


def config(layers, width=40, vocab=80, eps=2e-5, loop=None):
    c = {"architecture": "Bamudra", "width": width, "vocab": vocab, "norm": {"eps": eps},
         "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


FULL = config([attention(mlp=dense()), retention(mlp=dense(24, 1.7)),
               attention(heads=3, kv_heads=1, dim=10, rot_=rot(10, 9.0), size=5, keep=1),
               retention(heads=3, dim=16, vdim=4, rot_=rot(16, 500.0)),
               retention(heads=1, dim=4, vdim=20, decay=[0.995], mlp=dense(12, 0.5))],
              loop=(1, 4, 3))


def engine(c, w, device, dtype, max_tokens=512, live=4, block_size=8, **kw):
    cfg = config_from_hf(c)
    params = from_bamudra_state_dict(cfg, {k: torch.as_tensor(v) for k, v in w.items()}, dtype=dtype)
    return LLMEngine(cfg, device=device, dtype=dtype, params=params, max_batch=live,
                     max_model_len=1 << 20, block_size=block_size,
                     num_blocks=-(-max_tokens // block_size) + live,
                     use_graphs=kw.pop("graphs", False), lookahead=kw.pop("lookahead", False), **kw)


def tol(dtype):
    return 2e-4 if dtype == torch.float32 else 6e-2


def close(got, want, dtype, what="", slack=1.0):
    """Row error as a logit comparison sees it: mean removed, relative to the spread."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    err = np.sqrt((d ** 2).mean(-1)) / want.std()
    assert err.max() < slack * tol(dtype), \
        f"{what}: error {err.max():.3g} at row {int(err.argmax())}"


def replay(eng, tokens, cuts, rid="a"):
    """Feed ``tokens`` in portions ``cuts``; returns the logits of every position."""
    out, at = [], 0
    for n in cuts:
        last = at + n == len(tokens)
        lg = eng.replay_step([(rid, tokens[at:at + n])], [list(range(n))], [rid] if last else [])
        out.append(lg.float().cpu().numpy())
        at += n
    assert at == len(tokens)
    return np.concatenate(out)


def toks(n, vocab, seed=1):
    return np.random.default_rng(seed).integers(0, vocab, n).tolist()


def dev_t(a, device, dtype=torch.float32):
    return torch.as_tensor(np.asarray(a), dtype=dtype).to(device)


def i32(a, device):
    return torch.tensor(np.asarray(a), dtype=torch.int32, device=device)


def layer_params(c, w, device, dtype, i=0):
    from distributed_llm_inferencing_amd.models.mixers import derive_constants
    cfg = config_from_hf(c)
    params = from_bamudra_state_dict(cfg, {k: torch.as_tensor(v) for k, v in w.items()}, dtype=dtype)
    lp = {k[len(f"layers.{i}."):]: v.to(device) for k, v in params.items()
          if k.startswith(f"layers.{i}.")}
    derive_constants(cfg.layer_specs[i], lp, torch.device(device))
    return cfg.layer_specs[i], lp


def hidden(T, D, seed):
    return O.bf16_exact(np.random.default_rng(seed).standard_normal((T, D)))


# ------------------------------------------------------------------ single mechanisms (ops)
@pytest.mark.parametrize("device", ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)])
def test_rotation_table_at_near_and_far_positions(device):
    from distributed_llm_inferencing_amd.models.mixers import yarn_frequencies
    pos = [0, 1, 7, 4095, 1_000_003]
    for dims, base in ((2, 10.0), (14, 777.0), (64, 5e5)):
        f, _ = yarn_frequencies(dims, base)
        got = H.rotation_table(i32(pos, device), f.to(device)).cpu().numpy()
        ang = np.asarray(pos, np.float64)[:, None] * base ** (-2.0 * np.arange(dims // 2) / dims)
        np.testing.assert_allclose(got, np.concatenate([np.cos(ang), np.sin(ang)], 1), atol=2e-7)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("D", [40, 23])
def test_residual_add_with_bias_and_embedding_rows(device, dtype, D):
    """One launch: the stream takes a sublayer's output, its bias and the rows a loop pass adds,
    and leaves normed."""
    rng = np.random.default_rng(D)
    T, eps = 5, 1e-3
    x, y, x0 = (rng.standard_normal((T, D)) for _ in range(3))
    b, w = O.bf16_exact(rng.standard_normal(D)), O.bf16_exact(rng.standard_normal(D))
    for kw, new in ((dict(), x + y), (dict(bias=b), x + y + b), (dict(add=x0), x + y + x0),
                    (dict(bias=b, add=x0), x + y + b + x0)):
        xt = dev_t(x, device)
        kw = {k: dev_t(v, device, dtype if k == "bias" else torch.float32) for k, v in kw.items()}
        h = H.resadd_groupnorm(xt, dev_t(y, device), dev_t(w, device, dtype), 1, eps, **kw)
        a = 2e-5 if dtype == torch.float32 else 3e-2
        np.testing.assert_allclose(xt.cpu().numpy(), new, atol=2e-6, rtol=2e-6)
        np.testing.assert_allclose(h.float().cpu().numpy(), O.norm(new, w, eps), atol=a, rtol=a)
    xt = dev_t(x, device)                   # no sublayer output pending
    H.resadd_groupnorm(xt, None, dev_t(w, device, dtype), 1, eps, add=dev_t(x0, device))
    np.testing.assert_allclose(xt.cpu().numpy(), x + x0, atol=2e-6, rtol=2e-6)


ATTENTIONS = {
    "gqa": attention(), "one_head": attention(1, 1, 16, rot_=rot(16, 10.0)),
    "mqa": attention(6, 1, 4, rot_=rot(2), size=3, keep=5),
    "no_rotation": attention(3, 3, 6, rot_={"base": 10.0, "dims": 0}, keep=0),
    "odd_rotation": attention(2, 2, 7, rot_=rot(6), size=1, keep=2),
    "window_one": attention(2, 1, 8, size=1, keep=0),
    "all_kept": attention(2, 1, 8, size=4, keep=100),
    "matrix_core_32": attention(4, 2, 32, scale=0.2, rot_=rot(16, 900.0), size=13, keep=4),
    "matrix_core_64": attention(4, 1, 64, scale=0.13, rot_=rot(64, 900.0), size=37, keep=2),
    "matrix_core_128": attention(4, 2, 128, scale=0.09, rot_=rot(64, 900.0), size=30, keep=6)}


def attention_steps(spec, lp, h, cuts, device, dtype, eps, bs=4, seed=1):
    """The layer's output over portions ``cuts`` through pages in random order."""
    from distributed_llm_inferencing_amd.models.mixers import StepView, rope_attention_mixer
    T = h.shape[0]
    nblk = -(-T // bs)
    perm = np.random.default_rng(seed).permutation(nblk + 3)[:nblk]
    rows = (nblk + 3) * bs
    cache = (torch.full((rows, spec.kv_heads * spec.dim), 7.0, dtype=dtype, device=device),
             torch.full((rows, spec.kv_heads * spec.vdim), -5.0, dtype=dtype, device=device))
    got, at = [], 0
    for n in cuts:
        step = StepView(i32([0, n], device), n, i32(np.arange(at, at + n), device),
                        i32([perm[t // bs] * bs + t % bs for t in range(at, at + n)], device),
                        i32(perm[None], device), bs, None, at + n)
        got.append(rope_attention_mixer(spec, lp, dev_t(h[at:at + n], device, dtype), step, cache,
                                        eps).float().cpu().numpy())
        at += n
    return np.concatenate(got)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", list(ATTENTIONS))
def test_attention_through_shuffled_pages(device, dtype, name):
    """Biased projections, partial rotation, values tied to the unrotated keys, window and kept
    first tokens: whole, in portions and token by token through pages in any order."""
    lay = ATTENTIONS[name]
    T, D, eps = 61, 24, 1e-5
    c = config([lay], width=D)
    w = O.random_weights(c, lay["mixer"]["heads"])
    spec, lp = layer_params(c, w, device, dtype)
    h = hidden(T, D, 3)
    want = O.attention(h, w, "l0.mix.", lay["mixer"], eps) - w["l0.mix.o.b"]   # added with the residual
    if name in ("gqa", "matrix_core_32", "matrix_core_128"):
        # the bound sees each part: another rotation, window or set of kept tokens shows
        mask = lay["mixer"]["mask"]
        for k, v in (("rot", {"base": 10.0, "dims": 0}), ("mask", dict(mask, keep_first=0)),
                     ("mask", dict(mask, keep_first=mask["keep_first"] + 1)),
                     ("mask", dict(mask, size=mask["size"] + 1))):
            other = O.attention(h, w, "l0.mix.", dict(lay["mixer"], **{k: v}), eps) - w["l0.mix.o.b"]
            assert np.abs(other - want).max() > 0.1, (k, v)
    a = 2e-4 if dtype == torch.float32 else 5e-2
    for cuts in ([T], [5, 1, 2, T - 8], [1] * T, [33, 17, 11]):
        np.testing.assert_allclose(attention_steps(spec, lp, h, cuts, device, dtype, eps), want,
                                   atol=a, rtol=a, err_msg=str(cuts[:4]))


@pytest.mark.parametrize("device,dtype", CASES)
def test_attention_with_values_of_its_own(device, dtype):
    """The same mixer without tied values and without biases (another design's use of it)."""
    from dataclasses import replace
    T, D, eps = 30, 24, 1e-5
    lay = attention(4, 2, 8)
    c = config([lay], width=D)
    w = O.random_weights(c, 8)
    spec, lp = layer_params(c, w, device, dtype)
    rng = np.random.default_rng(4)
    wv = O.bf16_exact(rng.standard_normal((2 * 12, D)) / 5)
    wo = O.bf16_exact(rng.standard_normal((D, 4 * 12)) / 5)
    spec = replace(spec, vdim=12, tied_values=False, bias=False)
    lp = dict(lp, w_in=torch.cat([lp["w_in"], dev_t(wv, device, dtype)], 0), wo=dev_t(wo, device, dtype))
    del lp["b_in"], lp["b_out"]
    h = hidden(T, D, 3)
    q = O.rotate_half((h @ w["l0.mix.q"].T).reshape(T, 4, 8), np.arange(T), lay["mixer"]["rot"])
    k = O.rotate_half((h @ w["l0.mix.k"].T).reshape(T, 2, 8), np.arange(T), lay["mixer"]["rot"])
    v = (h @ wv.T).reshape(T, 2, 12)
    ok = O.visible(T, lay["mixer"]["mask"])
    o = np.zeros((T, 4, 12))
    for hh in range(4):
        sc = np.where(ok, q[:, hh] @ k[:, hh // 2].T * lay["mixer"]["scale"], -np.inf)
        e = np.exp(sc - sc.max(-1, keepdims=True))
        o[:, hh] = e / e.sum(-1, keepdims=True) @ v[:, hh // 2]
    a = 2e-4 if dtype == torch.float32 else 5e-2
    for cuts in ([T], [1] * T):
        np.testing.assert_allclose(attention_steps(spec, lp, h, cuts, device, dtype, eps),
                                   o.reshape(T, -1) @ wo.T, atol=a, rtol=a)


RETENTIONS = [(2, 8, 12, 4), (3, 5, 3, 2), (1, 16, 64, 16), (2, 32, 16, 8), (1, 64, 72, 64),
              (2, 128, 128, 128), (1, 48, 100, 16), (2, 16, 63, 0), (1, 96, 40, 0), (1, 256, 32, 128),
              (1, 32, 200, 24), (2, 16, 20, 12)]


def retention_run(spec, lp, hs, parts, cache, device, dtype, eps):
    """One step over parts [(name, slot, start, n)]; returns the rows of the layer's output."""
    from distributed_llm_inferencing_amd.models.mixers import StepView, retention_mixer
    rows = np.concatenate([hs[nm][s:s + n] for nm, _, s, n in parts])
    lens = [n for *_, n in parts]
    pos = np.concatenate([np.arange(s, s + n) for _, _, s, n in parts])
    step = StepView(i32(np.concatenate([[0], np.cumsum(lens)]), device), max(lens), i32(pos, device),
                    i32(pos, device), i32([[0]] * len(parts), device), 8,
                    i32([sl for _, sl, _, _ in parts], device), int(pos.max()) + 1)
    return retention_mixer(spec, lp, dev_t(rows, device, dtype), step, cache, eps).float().cpu().numpy()


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H_,d,dv,rd", RETENTIONS)
def test_retention_and_its_state(device, dtype, H_, d, dv, rd):
    """Portions of every length around a chunk's edge and single tokens of two interleaved
    sequences whose slots held stale states, against the oracle over each whole sequence."""
    D, eps = 24, 1e-5
    lay = retention(H_, d, dv, [1.0, 0.93, 0.8][:H_], rot(rd, 300.0))
    c = config([lay], width=D)
    w = O.random_weights(c, 5 + d)
    spec, lp = layer_params(c, w, device, dtype)
    hs = {"a": hidden(180, D, 1), "b": hidden(20, D, 2)}
    want = {k: O.retention(v, w, "l0.mix.", lay["mixer"], eps) for k, v in hs.items()}
    cache = (torch.full((3, H_, d, dv), 3.0, device=device),)
    a = 5e-4 if dtype == torch.float32 else 6e-2
    at = {"a": 0, "b": 0}
    slot = {"a": 2, "b": 0}
    for step in ([("a", 19), ("b", 1)], [("b", 1), ("a", 2)], [("a", 1), ("b", 7)], [("a", 64)],
                 [("a", 1)], [("b", 9), ("a", 70)], [("a", 16), ("b", 2)], [("a", 7)]):
        got = retention_run(spec, lp, hs, [(k, slot[k], at[k], n) for k, n in step], cache, device,
                            dtype, eps)
        o = 0
        for k, n in step:
            np.testing.assert_allclose(got[o:o + n], want[k][at[k]:at[k] + n], atol=a, rtol=a,
                                       err_msg=f"{k} at {at[k]}")
            o += n
            at[k] += n
    assert at == {"a": 180, "b": 20}
    assert float(cache[0][1].min()) == 3.0 and float(cache[0][1].max()) == 3.0


@pytest.mark.parametrize("device,dtype", CASES)
def test_retention_finds_one_far_key(device, dtype):
    """Every value but one is zero; that one lies hundreds of tokens (several chunks) back, under
    a decay of one: reading it needs the state carried over every chunk and portion."""
    D, eps, T, far = 24, 1e-6, 300, 5
    lay = retention(1, 16, 8, [1.0], rot(8, 300.0))
    c = config([lay], width=D)
    w = O.random_weights(c, 3)
    h = hidden(T, D, 5)
    null = np.linalg.svd(w["l0.mix.v"])[2][8:]                # inputs the value projection ignores
    keep = h[far].copy()
    h = h @ null.T @ null
    h[far] = keep
    want = O.retention(h, w, "l0.mix.", lay["mixer"], eps)
    spec, lp = layer_params(c, w, device, torch.float32)
    a = 2e-3
    for cuts in ([T], [64, 64, 128, 44], [3, 2, 1, 63, 65, 16, T - 150]):
        cache = (torch.full((1, 1, 16, 8), 9.0, device=device),)
        got, at = [], 0
        for n in cuts:
            got.append(retention_run(spec, lp, {"a": h}, [("a", 0, at, n)], cache, device,
                                     torch.float32, eps))
            at += n
        got = np.concatenate(got)
        assert np.abs(want[-20:]).max() > 0.2                 # the far value is what is read
        np.testing.assert_allclose(got[far:], want[far:], atol=a, rtol=a)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("ff,limit", [(40, 0.9), (7, 0.3), (64, 100.0), (192, 1.0)])
def test_clamped_feed_forward(device, dtype, ff, limit):
    from distributed_llm_inferencing_amd.models.mixers import FEED_FORWARDS
    D, T = 64, 33
    c = config([retention(mlp=dense(ff, limit))], width=D)
    w = O.random_weights(c, 7)
    spec, lp = layer_params(c, w, device, dtype)
    h = hidden(T, D, 9)
    got = FEED_FORWARDS[spec.ff_kind](spec, lp, dev_t(h, device, dtype)).cpu().numpy()
    a = 1e-4 if dtype == torch.float32 else 4e-2
    np.testing.assert_allclose(got, O.dense_ff(h, w, "l0.mlp.", limit), atol=a, rtol=a)
    g, u = h @ w["l0.mlp.gate"].T, h @ w["l0.mlp.up"].T
    if limit < 50:                                    # every clamp is active somewhere
        assert (g > limit).any() and (u > limit).any() and (u < -limit).any()


@pytest.mark.gpu
@pytest.mark.parametrize("M,splits", [(3, 2), (40, 4), (130, 2)])
def test_residual_add_sums_the_partial_sums_of_a_split_gemm(M, splits):
    from distributed_llm_inferencing_amd.ops import gemm as G
    N, K, eps = 192, 512, 1e-5
    x, w = hidden(M, K, 1), O.bf16_exact(hidden(N, K, 2) / 20)
    base, b, nw = hidden(M, N, 3), hidden(1, N, 4)[0], hidden(1, N, 5)[0]
    key = (G._bucket(M), N, K, "f32")
    old = G._plan_cache.get(key)
    G.set_plan(M, N, K, "f32", G.GemmPlan("dli", 0, splits))
    try:
        bf = torch.bfloat16
        xt, wt = dev_t(x, "cuda", bf), dev_t(w, "cuda", bf)
        y = H.linear_out(xt, wt)
        assert y.shape == (splits, M, N)
        st = dev_t(base, "cuda")
        h = H.resadd_groupnorm(st, y, dev_t(nw, "cuda", bf), 1, eps, bias=dev_t(b, "cuda", bf))
        want = base + x @ w.T + b
        np.testing.assert_allclose(st.cpu().numpy(), want, atol=2e-4, rtol=2e-4)
        np.testing.assert_allclose(h.float().cpu().numpy(), O.norm(want, nw, eps), atol=3e-2, rtol=3e-2)
        np.testing.assert_allclose(H.rows_of(H.linear_out(xt, wt)).cpu().numpy(), x @ w.T,
                                   atol=2e-4, rtol=2e-4)
    finally:
        G._plan_cache.pop(key, None) if old is None else G.set_plan(M, N, K, "f32", old)


@pytest.mark.gpu
@pytest.mark.parametrize("tile,splits", [(0, 1), (0, 2), (1, 4), (2, 1), (13, 1), (22, 1), (22, 2),
                                         (26, 1), (28, 2)])
@pytest.mark.parametrize("M", [5, 70, 300])
def test_clamped_swish_in_the_gemm_epilogue(tile, splits, M):
    from distributed_llm_inferencing_amd import ops
    from distributed_llm_inferencing_amd.ops import gemm as G
    from distributed_llm_inferencing_amd.ops.reference import interleave_gate_up
    F, K, lim = 448, 256, 0.8
    x, g, u = hidden(M, K, 1), O.bf16_exact(hidden(F, K, 2) / 12), O.bf16_exact(hidden(F, K, 3) / 12)
    bf = torch.bfloat16
    gu = interleave_gate_up(dev_t(g, "cuda", bf), dev_t(u, "cuda", bf)).contiguous()
    got = ops._gemm_native(dev_t(x, "cuda", bf), gu, "clamp_mul",
                           bias=torch.full((1,), lim, device="cuda"), plan=G.GemmPlan("dli", tile, splits))
    w = {"gate": g, "up": u, "down": np.eye(F)}
    want = O.dense_ff(x, w, "", lim)
    np.testing.assert_allclose(got.float().cpu().numpy(), want, atol=2e-2, rtol=2e-2)


# ------------------------------------------------------------------ whole models
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("lay", [retention(), retention(mlp=dense()), attention(),
                                 attention(mlp=dense())],
                         ids=["retention", "retention_dense", "attention", "attention_dense"])
@pytest.mark.parametrize("times", [0, 1, 2])
def test_one_layer_models(lay, times, device, dtype):
    c = config([lay], loop=(0, 1, times) if times else None)
    w = O.random_weights(c, 11)
    t = toks(21, c["vocab"])
    close(replay(engine(c, w, device, dtype), t, [21]), O.forward(c, w, t), dtype, "one layer")


@pytest.mark.parametrize("device,dtype", CASES)
def test_layer_trace_matches_the_oracle(device, dtype):
    w = O.random_weights(FULL, 2)
    t = toks(14, FULL["vocab"], 4)
    trace = []
    O.forward(FULL, w, t, trace)
    eng = engine(FULL, w, device, dtype)
    eng.model.layer_trace = []
    replay(eng, t, [14])
    assert len(eng.model.layer_trace) == len(trace) == 11          # 1 + 3 * 3 + 1 runs
    for i, (got, want) in enumerate(zip(eng.model.layer_trace, trace)):
        d = np.abs(got.cpu().numpy() - want).max()
        assert d < (1e-3 if dtype == torch.float32 else 3e-2 * np.abs(want).max()), f"run {i}"


@pytest.mark.parametrize("device,dtype", CASES)
def test_prefill_equals_decode_equals_portions(device, dtype):
    w = O.random_weights(FULL, 1)
    t = toks(45, FULL["vocab"], 3)
    want = O.forward(FULL, w, t)
    for cuts in ([45], [1] * 45, [2] * 22 + [1], [7, 2, 9, 1, 1, 3, 16, 2, 4],
                 [30] + [1] * 15, [8, 8, 8, 8, 8, 5], [17, 16, 12]):
        close(replay(engine(FULL, w, device, dtype), t, cuts), want, dtype, f"cuts {cuts[:4]}")


@pytest.mark.parametrize("device,dtype", CASES)
def test_mixed_batches_and_reuse_of_pages_and_slots(device, dtype):
    """Unequal requests in one step (portions beside single tokens) against each alone, in a
    pool so small that pages and state slots are freed and taken again."""
    w = O.random_weights(FULL, 4)
    V = FULL["vocab"]
    seqs = {k: toks(n, V, s) for k, n, s in (("a", 30, 1), ("b", 9, 2), ("c", 17, 3), ("d", 5, 4),
                                             ("e", 26, 5), ("f", 12, 6))}
    want = {k: O.forward(FULL, w, t) for k, t in seqs.items()}
    eng = engine(FULL, w, device, dtype, max_tokens=88, live=3)
    plan = [[("a", 6), ("b", 1)], [("a", 1), ("b", 2), ("c", 17)], [("a", 10), ("b", 6)],
            [("a", 13), ("d", 2)], [("d", 3), ("e", 20)], [("e", 1), ("f", 1)],
            [("e", 5), ("f", 9)], [("f", 2)]]
    at = {k: 0 for k in seqs}
    got = {k: [] for k in seqs}
    for step in plan:
        entries, wantidx, end = [], [], []
        for k, n in step:
            entries.append((k, seqs[k][at[k]:at[k] + n]))
            wantidx.append(list(range(n)))
            at[k] += n
            if at[k] == len(seqs[k]):
                end.append(k)
        lg = eng.replay_step(entries, wantidx, end).float().cpu().numpy()
        o = 0
        for k, n in step:
            got[k].append(lg[o:o + n])
            o += n
    for k in seqs:
        assert at[k] == len(seqs[k])
        close(np.concatenate(got[k]), want[k], dtype, f"request {k}")
    assert eng.bm.num_free == eng.bm.num_blocks and eng.state_slots.num_free == 3


@pytest.mark.parametrize("device,dtype", CASES)
def test_other_sizes_and_degenerate_values(device, dtype):
    """Sizes that differ where a usual model makes them equal, values of 1, no loop, a loop of one
    pass, a loop over everything, one kind of layer only, nothing a multiple of 4."""
    cs = [
        config([attention(1, 1, 4, 1.0, rot(2), 1, 1, dense(7, 1.0)), retention(1, 3, 5, [1.0], rot(2))],
               width=20, vocab=31),
        config([retention(5, 4, 2, rot_=rot(4, 3.0)), attention(6, 3, 2, rot_=rot(2), size=2, keep=0),
                attention(2, 1, 6, rot_=rot(2), size=30, keep=2, mlp=dense(9))],
               width=28, vocab=40, loop=(0, 3, 2)),
        config([attention(mlp=dense()), retention()], width=64, vocab=50, eps=1e-2, loop=(1, 2, 1)),
        config([attention(3, 1, 6, rot_=rot(2), size=4, keep=7, mlp=dense(5)),
                retention(3, 5, 7, rot_=rot(2), mlp=dense(9)), retention(1, 7, 9, [0.5], rot(6))],
               width=30, vocab=33, loop=(1, 3, 3)),
        config([retention(2, 16, 16, mlp=dense(12)), retention(2, 16, 8)], width=32, vocab=37),
        config([attention(2, 2, 16, rot_=rot(8)), attention(4, 1, 8, rot_={"dims": 0, "base": 9.0})],
               width=32, vocab=37, loop=(0, 1, 4)),
    ]
    for n, c in enumerate(cs):
        w = O.random_weights(c, 20 + n)
        t = toks(19, c["vocab"], n)
        want = O.forward(c, w, t)
        eng = engine(c, w, device, dtype, block_size=4)
        close(replay(eng, t, [19]), want, dtype, f"config {n} whole")
        close(replay(eng, t, [3, 1, 2, 13]), want, dtype, f"config {n} portions")


def standout_model(rotated, size=16, keep=3):
    """One attention layer whose last query finds one key: token 61's key is 1.6 times token
    62's query (keys share the query projection and bias), so it outscores every other key,
    the query's own included; its value, the key itself, is what the output then shows.
    ``rotated``: part of every head turns with the position, with small weights, so that the
    standing out survives any distance."""
    c = config([attention(2, 2, 4, 1.6, rot(2, 40.0) if rotated else {"base": 9.0, "dims": 0}, size,
                          keep)], width=32, vocab=64)
    w = O.random_weights(c, 9)
    if rotated:
        for hh in range(2):
            w["l0.mix.q"][hh * 4:hh * 4 + 2] *= 0.125
            w["l0.mix.q.b"][hh * 4:hh * 4 + 2] *= 0.125
    w["l0.mix.q"] *= 1.5
    w["l0.mix.q"] = O.bf16_exact(w["l0.mix.q"])
    w["l0.mix.k"], w["l0.mix.k.b"] = w["l0.mix.q"].copy(), w["l0.mix.q.b"].copy()
    w["l0.mix.o"] = w["l0.mix.o"] * 2.0                   # the mixer outweighs the residual
    A = w["l0.mix.q"] * w["l0.norm1"][None, :]            # what a key sees of the unit-RMS input
    x62 = O.rms(w["embed"][62], c["norm"]["eps"])
    key = 1.6 * (A @ x62 + w["l0.mix.q.b"]) - w["l0.mix.q.b"]
    x = np.linalg.pinv(A) @ key
    null = np.linalg.svd(A)[2][A.shape[0]:]
    rest = null.T @ np.random.default_rng(3).standard_normal(null.shape[0])
    left = 32.0 - (x ** 2).sum()
    assert left > 0
    w["embed"][61] = O.bf16_exact(x + rest * np.sqrt(left / (rest ** 2).sum()))
    return c, w


# (place of the standing-out key, length of the sequence, seen): window of 16, 3 kept tokens
EDGES = [(44, 60, True), (43, 60, False), (42, 60, False), (2, 60, True), (3, 60, False),
         (0, 60, True), (4, 60, False), (0, 300, True), (2, 300, True), (3, 300, False),
         (58, 60, True), (51, 60, True), (3, 19, True), (3, 20, False), (2, 19, True), (0, 2, True),
         (7, 9, True), (8, 9, True), (7, 23, True), (7, 24, False), (47, 63, True), (48, 64, True)]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("rotated", [False, True])
def test_keys_at_the_edges_of_the_window_and_the_kept_tokens(rotated, device, dtype):
    """One key dominates the last query's scores if it is seen: just inside and just outside the
    window and the kept first tokens, at page borders, far away; in a prompt, decoded, and with
    the portion cut at the key."""
    c, w = standout_model(rotated)
    for at, n, seen in EDGES:
        t = toks(n, 60, at + n)
        t[-1] = 62
        if at != n - 1:
            t[at] = 61
        want = O.forward(c, w, t)
        t2 = list(t)
        t2[at] = 60
        if at != n - 1:
            moved = np.abs(O.forward(c, w, t2)[-1] - want[-1]).max()
            assert (moved > 0.25) if seen else (moved == 0.0), (at, n, moved)
        eng = engine(c, w, device, dtype)
        what = f"key {at} of {n}"
        close(replay(eng, t, [n])[-1:], want[-1:], dtype, what + " whole")
        tail = min(n - 1, 17)
        close(replay(eng, t, [n - tail] + [1] * tail)[-1:], want[-1:], dtype, what + " decoded")
        cuts = [x for x in (at, 1, n - 2 - at, 1) if x > 0]
        if sum(cuts) == n:
            close(replay(eng, t, cuts)[-1:], want[-1:], dtype, what + " cut at the key")


@pytest.mark.parametrize("device,dtype", CASES)
def test_first_tokens_and_long_decode(device, dtype):
    w = O.random_weights(FULL, 6)
    t = toks(150, FULL["vocab"], 8)
    want = O.forward(FULL, w, t)
    eng = engine(FULL, w, device, dtype)
    got = replay(eng, t, [1, 1, 1, 2] + [1] * 145)
    close(got[:6], want[:6], dtype, "first tokens")
    close(got, want, dtype, "long decode", slack=1.0 if dtype == torch.float32 else 1.5)
    # the same slot and pages again, starting from a stale state
    t2 = toks(12, FULL["vocab"], 9)
    close(replay(eng, t2, [1] * 12), O.forward(FULL, w, t2), dtype, "reused")


@pytest.mark.parametrize("device,dtype,graphs", [
    ("cpu", torch.float32, False),
    pytest.param("cuda", torch.float32, False, marks=pytest.mark.gpu),
    pytest.param("cuda", torch.bfloat16, True, marks=pytest.mark.gpu)])
def test_greedy_generation_through_the_engine(device, dtype, graphs):
    """``LLMEngine.generate``: scheduler, chunked prefill, decode steps (captured graphs and
    lookahead on the GPU) against greedy decoding with the oracle; several batches, so that
    captured steps are replayed for other requests, pages and slots."""
    c = FULL
    w = O.random_weights(c, 12)
    w["head"] = w["head"] * 4.0                          # clear winners
    eng = engine(c, w, device, dtype, graphs=graphs, lookahead=graphs, max_prefill_tokens=16)
    for batch in (((11, 1), (3, 2), (25, 3)), ((30, 4), (2, 5)), ((7, 6), (18, 7), (1, 8))):
        prompts = [toks(n, c["vocab"], s) for n, s in batch]
        outs = eng.generate(prompts, SamplingParams(max_new_tokens=8, do_sample=False,
                                                    ignore_eos=True))
        for p, o in zip(prompts, outs):
            seq = list(p)
            assert len(o.output_ids) == 8
            for tok in o.output_ids:
                lg = O.forward(c, w, seq)[-1]
                best = int(lg.argmax())
                if tok != best:          # a near tie may fall the other way in reduced precision
                    assert lg[best] - lg[tok] < (1e-3 if dtype == torch.float32 else 0.3)
                seq.append(tok)


def test_config_reader_reads_every_size():
    cfg = config_from_hf(FULL)
    assert cfg.arch == "bamudra" and cfg.is_hybrid and cfg.has_state
    assert (cfg.hidden_size, cfg.vocab_size, cfg.norm_eps) == (40, 80, 2e-5)
    assert cfg.loop == (1, 4, 3) and cfg.loop_add and not cfg.loop_entry
    assert [li for li, _, _ in cfg.layer_runs()] == [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4]
    s = cfg.layer_specs
    assert [x.kind for x in s] == ["rope_attention", "retention", "rope_attention", "retention",
                                   "retention"]
    assert (s[0].heads, s[0].kv_heads, s[0].dim, s[0].vdim, s[0].scale, s[0].rot_dims, s[0].rot_base,
            s[0].window, s[0].keep_first) == (4, 2, 8, 8, 0.45, 6, 60.0, 11, 3)
    assert s[0].bias and s[0].tied_values
    assert (s[0].ff, s[0].ff_kind, s[0].act_limit) == (40, "clamp_swish", 0.9)
    assert (s[3].heads, s[3].dim, s[3].vdim, s[3].rot_dims, s[3].rot_base, s[3].ff) == (3, 16, 4, 16, 500.0, 0)
    assert len(s[3].decays) == 3
    assert cfg.cache_row_width(0) == 2 * 16 and cfg.cache_row_width(1) == 0
    # the configuration survives the dictionary form the workers exchange
    from distributed_llm_inferencing_amd.models.configs import ModelConfig
    assert ModelConfig.from_dict(cfg.to_dict()) == cfg
    sd = {k: torch.as_tensor(v) for k, v in O.random_weights(FULL, 0).items()}
    params = from_bamudra_state_dict(cfg, sd)
    assert params["layers.0.w_in"].shape == ((4 + 2) * 8, 40)
    assert params["layers.1.w_in"].shape == (2 * 2 * (8 + 12), 40)
    # no mask: every earlier position; no loop: nothing is added
    c = config([attention()])
    del c["layers"][0]["mixer"]["mask"]
    cfg = config_from_hf(c)
    assert cfg.layer_specs[0].window == 1 << 30 and not cfg.loop and not cfg.loop_add
    for path, v in ((("mixer", "decay"), [0.5]), (("mixer", "rot", "dims"), 3),
                    (("mixer", "rot", "dims"), 10), (("mlp", "kind"), "moe")):
        bad = copy.deepcopy(FULL)
        o = bad["layers"][1]
        for k in path[:-1]:
            o = o[k]
        o[path[-1]] = v
        with pytest.raises(ValueError):
            config_from_hf(bad)
    bad = dict(sd)
    bad["l1.mix.v"] = bad["l1.mix.v"][:-1]
    with pytest.raises(ValueError):
        from_bamudra_state_dict(config_from_hf(FULL), bad)


def test_registry_model_random_init_generates():
    eng = LLMEngine("bamudra-tiny", device="cpu", dtype=torch.float32, max_batch=2,
                    max_model_len=64, block_size=8, num_blocks=24, use_graphs=False)
    outs = eng.generate([[1, 2, 3], [4, 5, 6, 7, 8]], SamplingParams(max_new_tokens=4, do_sample=False,
                                                                    ignore_eos=True))
    assert all(len(o.output_ids) == 4 for o in outs)


@pytest.mark.gpu
@pytest.mark.parametrize("width,lay,n", [
    (128, retention(2, 64, 128, [0.97, 0.999], rot(32), dense(192)), 150),
    (192, retention(2, 128, 64, [0.9, 1.0], rot(128, 5000.0), dense(128)), 201),
    (128, attention(6, 2, 64, 0.11, rot(48, 800.0), 53, 4, dense(256)), 333),
    (192, attention(8, 2, 128, 0.09, rot(128, 3000.0), 100, 5, dense(64)), 410),
    (64, attention(16, 1, 128, 0.09, rot(64, 3000.0), 300, 1), 700)],
    ids=["retention_64", "retention_128", "attention_64", "attention_128", "attention_16_heads"])
def test_matrix_core_sizes_at_length(width, lay, n):
    """Sizes that the matrix-core kernels and the tuned GEMM tiles take: whole prompts, portions
    and single tokens over long contexts, alone and several at once."""
    c = config([lay, lay], width=width, vocab=96)
    w = O.random_weights(c, width + n)
    t, t2, t3 = toks(n, 96, n), toks(n // 2, 96, 2), toks(40, 96, 3)
    want, want2, want3 = (O.forward(c, w, x) for x in (t, t2, t3))
    eng = engine(c, w, "cuda", torch.bfloat16, max_tokens=2 * n + 64, block_size=16)
    bf = torch.bfloat16
    close(replay(eng, t, [n]), want, bf, "whole")
    close(replay(eng, t, [n - 9, 2, 1, 1, 5]), want, bf, "portions")
    close(replay(eng, t, [n - 20] + [1] * 20), want, bf, "decoded")
    m = n // 2
    lg = eng.replay_step([("a", t[:n - 30]), ("b", t2[:m - 3]), ("c", t3[:37])],
                         [[n - 31], [0, m - 4], [36]]).float().cpu().numpy()
    close(lg, np.stack([want[n - 31], want2[0], want2[m - 4], want3[36]]), bf, "together")
    for i in range(3):
        lg = eng.replay_step([("a", t[n - 30 + i:n - 29 + i]), ("b", t2[m - 3 + i:m - 2 + i]),
                              ("c", t3[37 + i:38 + i])], [[0], [0], [0]],
                             ["b", "c"] if i == 2 else []).float().cpu().numpy()
        close(lg, np.stack([want[n - 30 + i], want2[m - 3 + i], want3[37 + i]]), bf, "singles together")
    lg = eng.replay_step([("a", t[n - 27:])], [list(range(27))], ["a"]).float().cpu().numpy()
    close(lg, want[n - 27:], bf, "last portion")


def test_checkpoint_folder_through_the_replay_command(tmp_path, monkeypatch, capsys):
    """A checkpoint folder (config.json + model.safetensors in bfloat16) read by the C++
    safetensors loader, and the trace replay command driving the engine: two requests in mixed
    steps, logits written per step."""
    import io
    import json
    from safetensors.torch import save_file
    from distributed_llm_inferencing_amd.cli import main as cli_main
    c = config([retention(mlp=dense()), attention(mlp=dense())], loop=(0, 2, 2))
    w = O.random_weights(c, 21)
    model = tmp_path / "model"
    model.mkdir()
    (model / "config.json").write_text(json.dumps(c))
    save_file({k: torch.as_tensor(v).to(torch.bfloat16).contiguous() for k, v in w.items()},
              str(model / "model.safetensors"))
    ta, tb = toks(21, c["vocab"], 1), toks(9, c["vocab"], 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": ta[:13], "want": [0, 12]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": ta[13:14], "want": [0]},
                                     {"id": "b", "tokens": tb, "want": [3, 8]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": ta[14:], "want": []}], "end": ["a"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n"))
    out = tmp_path / "out"
    rc = cli_main(["trace-run", "--model", str(model), "--dtype", "float32", "--out", str(out),
                   "--max-tokens", "128", "--device", "cpu"])
    assert rc == 0
    assert [ln for ln in capsys.readouterr().out.splitlines() if ln.startswith("done")] == \
        ["done 0", "done 1", "done 2"]
    ra, rb = O.forward(c, w, ta), O.forward(c, w, tb)
    V = c["vocab"]
    got0 = np.fromfile(out / "0.f32", dtype="<f4").reshape(-1, V)
    got1 = np.fromfile(out / "1.f32", dtype="<f4").reshape(-1, V)
    close(got0, ra[[0, 12]], torch.float32, "step 0")
    close(got1, np.stack([ra[13], rb[3], rb[8]]), torch.float32, "step 1")
    assert not (out / "2.f32").exists()
