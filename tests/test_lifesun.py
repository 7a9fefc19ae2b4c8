"""The Lifesun design in the engine against its plain implementation (``plain_lifesun.py``): every mechanism alone,
then whole models however the requests are cut and batched, on the plain ops (CPU) and on the HIP kernels (GPU)."""
import collections
import json
import os
import subprocess
import sys
import types

import numpy as np
import pytest
import torch

import plain_lifesun as P
import traces
from lifesun_configs import LIFESUN, LIFESUN_FAST, draw_lifesun, lifesun_config_json, write_lifesun
from jax_llm_examples_amd import Engine, SamplingParams, load_model
from jax_llm_examples_amd.cache import CacheManager, CacheView
from jax_llm_examples_amd.config import ConfigError, get_architecture
from jax_llm_examples_amd.config.specs import part
from jax_llm_examples_amd.engine import StepEntry, build_context, get_ops
from jax_llm_examples_amd.engine.replay import make_runner
from jax_llm_examples_amd.parts.base import Rotation, build_head, build_norm
from jax_llm_examples_amd.parts.loop import build_loop
from jax_llm_examples_amd.parts.residual import Residual, ScaledSum

DEVICES = [pytest.param("cpu", id="cpu-plain-ops"), pytest.param("cuda:0", id="gpu-hip", marks=pytest.mark.gpu)]
DTYPED = [pytest.param("cpu", torch.float32, id="cpu-plain-ops"),
          pytest.param("cuda:0", torch.float32, id="gpu-f32", marks=pytest.mark.gpu),
          pytest.param("cuda:0", torch.bfloat16, id="gpu-bf16", marks=pytest.mark.gpu)]
LENGTHS = {"LA": [1, 80, 33, 47, 64, 9, 130], "LB": [70, 2, 49, 96, 31, 17], "LS": [161, 40, 5, 83],
           "LF": [420, 40, 170, 33, 128], "LW": [290, 40, 129, 17]}
MODES = {"whole": traces.whole, "tail": traces.tail, "portions": traces.portions, "mixed": traces.mixed}
TOL = {"float32": 5e-5, "bfloat16": 5e-2}  # of the largest logit of the request
# (in bfloat16 also three times what weights that are off by up to 2^-8 do to a position: a retention head whose first
# query and key are nearly orthogonal is a matter of sign, and sharp scores move weights by more than they are rounded)


def _ops(device):
    return get_ops(device, reference_ops=(device == "cpu"))


def _load(folder, dtype, device):
    if device != "cpu":
        return load_model(folder, dtype, device)
    from jax_llm_examples_amd.engine.loading import load_model as lm
    return lm(folder, dtype, "cpu")


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("lifesun")
    return {name: write_lifesun(name, str(root / name), torch.float32) for name in LIFESUN}


@pytest.fixture(scope="module")
def folders_bf16(tmp_path_factory):
    root = tmp_path_factory.mktemp("lifesun_bf16")
    return {name: write_lifesun(name, str(root / name), torch.bfloat16) for name in {**LIFESUN, **LIFESUN_FAST}}


def _doubles(w):
    return {k: v.double() for k, v in w.items() if v.is_floating_point()}


# ---------------------------------------------------------------------------------------------- norm, sums, loop, head
@pytest.mark.parametrize("device,dtype", DTYPED)
@pytest.mark.parametrize("width", [37, 54, 256, 300, 1000, 1028, 4096, 8200, 20000, 5001])
def test_layer_norm_of_a_sum_of_terms(device, dtype, width):
    """Up to three weighted terms join the residual (float32) and the layer norm's rows come out of the same call; rows
    with a large mean (the variance is that of the deviations) and every width class of the kernel."""
    norm = build_norm(part("layernorm", eps=1e-3, size=width))
    norm.allocate(torch.float32, torch.device(device))
    g = torch.Generator().manual_seed(width)
    w, b = torch.rand(width, generator=g) + 0.5, torch.randn(width, generator=g)
    norm.params["weight"].copy_(w)
    norm.params["bias"].copy_(b)
    ctx = types.SimpleNamespace(ops=_ops(device), dtype=dtype, device=torch.device(device))
    for count in (0, 1, 2, 3):
        x = torch.randn(5, width, generator=g) + 30.0
        terms = [(torch.randn(5, width, generator=g).to(dtype), f) for f in (0.7, -1.3, 2.0)[:count]]
        want_x = x.double() + sum((f * t.double() for t, f in terms), torch.zeros(5, width, dtype=torch.float64))
        r = Residual(x.to(device))
        if terms:
            r.add(ScaledSum([(t.to(device), f) for t, f in terms]))
        h, h32 = norm.forward(r, ctx, want32=True)
        want = P.layer_norm(want_x, w.double(), b.double(), 1e-3)
        assert h.dtype == dtype
        assert torch.allclose(h32.cpu().double(), want, rtol=1e-4, atol=2e-5), (h32.cpu().double() - want).abs().max()
        assert torch.equal(h.cpu(), h32.cpu().to(dtype))
        assert torch.allclose(r.value(ctx).cpu().double(), want_x, rtol=1e-6, atol=1e-5)


@pytest.mark.parametrize("device", DEVICES)
def test_three_terms_elsewhere(device):
    """A sum of three terms that is asked for as a value, for some rows, or through a root-mean-square norm."""
    g = torch.Generator().manual_seed(2)
    x, idx = torch.randn(6, 80, generator=g), torch.tensor([4, 1], dtype=torch.int32)
    terms = [(torch.randn(6, 80, generator=g), f) for f in (0.5, 2.0, -1.0)]
    total = x.double() + sum(f * t.double() for t, f in terms)
    ctx = types.SimpleNamespace(ops=_ops(device), dtype=torch.float32, device=torch.device(device))
    fresh = lambda: ScaledSum([(t.to(device), f) for t, f in terms])
    r = Residual(x.clone().to(device))
    r.add(fresh())
    some = r.rows(ctx, idx.to(device))
    assert torch.allclose(some.value(ctx).cpu().double(), total[[4, 1]], atol=1e-5)
    h, _ = r.normed(ctx, None, 1e-5)
    assert torch.allclose(h.cpu().double(), P.rms_divide(total, 1e-5), atol=1e-5)
    assert torch.allclose(ctx.ops.materialize(fresh()).cpu().double(), total - x.double(), atol=1e-5)


@pytest.mark.parametrize("device,dtype", DTYPED)
@pytest.mark.parametrize("width,tokens", [(50, 3), (64, 1), (256, 20), (1280, 70), (96, 300)])
def test_pass_projection_alone(device, dtype, width, tokens):
    """``W [x; x0]`` with a branch output still pending on x: the result is float32-precise in x also in bfloat16 (a
    stream rounded to bfloat16 on its way would be off by 2^-9)."""
    loop = build_loop(part("pass_projection", hidden_size=width, times=2))
    loop.allocate(dtype, torch.device(device))
    g = torch.Generator().manual_seed(width + tokens)
    w = (torch.randn(width, 2 * width, generator=g) / (2 * width) ** 0.5).to(dtype)
    loop.params["weight"].copy_(w)
    loop.finalize()
    x0 = torch.randn(tokens, width, generator=g).to(dtype).float()
    x, y = torch.randn(tokens, width, generator=g) * 3.0, torch.randn(tokens, width, generator=g).to(dtype)
    ctx = types.SimpleNamespace(ops=_ops(device), dtype=dtype, device=torch.device(device))
    r = Residual(x.to(device))
    r.add(ScaledSum([(y.to(device), 0.5)]))
    loop.enter(r, x0.to(device), 0, ctx)
    want = torch.cat([x.double() + 0.5 * y.double(), x0.double()], dim=1) @ w.double().T
    got = r.value(ctx)
    assert got.dtype == torch.float32
    tol = 1e-4 if dtype == torch.bfloat16 else 2e-5
    assert (got.cpu().double() - want).abs().max() < tol, (got.cpu().double() - want).abs().max()
    with pytest.raises(ValueError):
        loop.enter(r, x0.to(device), 2, ctx)


@pytest.mark.parametrize("device", DEVICES)
def test_head_with_a_scale(device):
    head = build_head(part("linear_head", vocab_size=70, hidden_size=48, scale=0.37))
    head.allocate(torch.float32, torch.device(device))
    g = torch.Generator().manual_seed(3)
    w, h = torch.randn(70, 48, generator=g), torch.randn(4, 48, generator=g)
    head.params["weight"].copy_(w)
    head.finalize()
    got = head.forward(h.to(device), types.SimpleNamespace(ops=_ops(device)), None)
    assert torch.allclose(got.cpu().double(), 0.37 * h.double() @ w.double().T, rtol=1e-5, atol=1e-5)


# ---------------------------------------------------------------------------------------------- the two recurrences
def _step_arrays(lengths, extra, device, g, starts=None):
    bounds, o = [], 0
    for n in lengths:
        bounds.append((o, o + n))
        o += n
    slots = torch.randperm(len(lengths) + extra, generator=g)[: len(lengths)]
    phase = torch.randint(0, 2, (len(lengths),), generator=g)
    starts = starts or [0] * len(lengths)
    pos = torch.cat([torch.arange(s, s + n) for s, n in zip(starts, lengths)])
    d = lambda t: t.to(device)
    ctx = types.SimpleNamespace(cu_seqlens=d(torch.tensor([0] + [b for _, b in bounds], dtype=torch.int32)),
                                state_slots=d(slots.int()), state_phase=d(phase.int()), num_segments=len(lengths),
                                seg_lens=list(lengths), num_tokens=o, positions=d(pos.int()), scratch={})
    return bounds, slots, phase, pos, ctx


def _left_behind(st, state, slots, phase, left, tol):
    """The other halves hold the new memory, and nothing else was written."""
    st = st.cpu()
    new = st[slots, 1 - phase].double()
    assert (new - left).abs().max() < tol * left.abs().max(), (new - left).abs().max() / left.abs().max()
    st[slots, 1 - phase] = state[slots, 1 - phase]
    assert torch.equal(st, state)


@pytest.mark.parametrize("device,dtype", DTYPED)
@pytest.mark.parametrize("W,blocks,lengths", [
    (256, 2, [64, 1, 65, 63, 130]), (192, 12, [200, 2, 128]), (48, 3, [5, 70]), (35, 7, [33, 129]), (128, 4, [1, 1, 1]),
    (300, 1, [90, 15]), (1024, 2, [66]), (72, 2, [16, 17, 31, 32, 48, 12]), (512, 4, [1] * 40), (96, 1, [1] * 20),
    (13, 13, [300]), (21, 3, [1] * 5)])
def test_gated_unit_alone(device, dtype, W, blocks, lengths):
    """Segments that end before, at and behind a chunk's edge and steps of single tokens, from a memory that is not zero,
    with decays that forget within a token beside ones that keep thousands; the outputs and, much sharper, the memory
    that is left, against float64.  The memory is as a float32 recurrence leaves it in either run dtype."""
    g = torch.Generator().manual_seed(W * 10 + blocks)
    N, s = sum(lengths), W // blocks
    rnd = lambda *sh: torch.randn(*sh, generator=g)
    u, wide = rnd(N, W).to(dtype), rnd(N, 2 * W).to(dtype)  # (the other branch lies in wider rows)
    yb, bra, bri = rnd(W) * 0.3, rnd(blocks, s) * 2.0, rnd(blocks, s)
    wra, wri = (rnd(blocks, s, s) * s ** -0.5).to(dtype), (rnd(blocks, s, s) * s ** -0.5).to(dtype)
    lam = torch.linspace(-12.0, 3.0, W)[torch.randperm(W, generator=g)]
    bounds, slots, phase, _, ctx = _step_arrays(lengths, 2, device, g)
    state = rnd(len(lengths) + 2, 2, W)
    ud = u.double().view(N, blocks, s)
    sig = lambda w, b: torch.sigmoid(torch.einsum("nbk,bok->nbo", ud, w.double()) + b.double()).reshape(N, W)
    log_a = -8.0 * sig(wra, bra) * torch.nn.functional.softplus(lam.double())
    take = torch.sqrt(-torch.expm1(2 * log_a)) * sig(wri, bri) * u.double()
    want, left = torch.zeros(N, W, dtype=torch.float64), []
    for i, (lo, hi) in enumerate(bounds):
        S = state[slots[i], phase[i]].double()
        for t in range(lo, hi):
            S = torch.exp(log_a[t]) * S + take[t]
            want[t] = S
        left.append(S)
    want = want * P.gelu_tanh(wide[:, W:].double() + yb.double())
    d = lambda t: t.to(device)
    st = d(state.clone())
    got = _ops(device).gated_unit(d(u), d(wide)[:, W:], d(yb), d(wra), d(bra), d(wri), d(bri), d(lam), 8.0, st, ctx)
    tol = 1e-2 if dtype == torch.bfloat16 else 1e-4
    assert got.dtype == dtype and torch.allclose(got.cpu().double(), want, rtol=tol, atol=tol), (got.cpu().double() - want).abs().max()
    _left_behind(st, state, slots, phase, torch.stack(left), 2e-5)


def _retained(rows, H, dk, dv, rot, decay, eps, pos, state, bounds):
    """float64, token by token; ``state`` [segments, H, dv, dk] in front of the segments."""
    r = rows.double()
    N = r.shape[0]
    q, k = r[:, : H * dk].reshape(N, H, dk), r[:, H * dk: 2 * H * dk].reshape(N, H, dk)
    if rot is not None:
        q, k = P.turn(q, pos.tolist(), rot), P.turn(k, pos.tolist(), rot)
    k, v = k * dk ** -0.5, r[:, 2 * H * dk: 2 * H * dk + H * dv].reshape(N, H, dv)
    out, left = torch.zeros(N, H, dv, dtype=torch.float64), []
    dec = torch.tensor(decay, dtype=torch.float64)[:, None, None]
    for i, (lo, hi) in enumerate(bounds):
        S = state[i].double().clone()
        for t in range(lo, hi):
            S = dec * S + v[t][:, :, None] * k[t][:, None, :]
            out[t] = (S * q[t][:, None, :]).sum(-1)
        left.append(S)
    return P.rms_divide(out, eps).reshape(N, H * dv) * P.silu(r[:, 2 * H * dk + H * dv:]), torch.stack(left)


def _rotation(rot, dk, device):
    if rot is None:
        return None
    inv = torch.tensor([rot["base"] ** (-2.0 * i / rot["dims"]) for i in range(rot["dims"] // 2)], dtype=torch.float64)
    return Rotation(inv.float().to(device), pairing="half", rotary_dim=rot["dims"])


def _decays(decay, device):
    g = torch.tensor(decay, dtype=torch.float32)
    return torch.stack([g, torch.log2(g.double()).clamp_min(-1e6).float()]).to(device)


@pytest.mark.parametrize("device,dtype", DTYPED)
@pytest.mark.parametrize("H,dk,dv,dims,decay,lengths", [
    (3, 64, 64, 64, [0.5, 0.984375, 0.9995], [128, 1, 129, 127, 260]), (2, 128, 256, 64, [0.97, 1.0], [300, 2, 16]),
    (2, 20, 24, 12, [0.9, 0.0], [5, 150]), (1, 6, 10, 4, [0.99], [33, 257]), (2, 40, 72, None, [0.999, 0.7], [1, 1, 1]),
    (1, 256, 512, 256, [0.998], [140, 15]), (2, 72, 130, 72, [0.95, 0.9999], [66]), (1, 300, 33, 8, [0.9], [20, 3]),
    (4, 96, 64, 2, [0.1, 0.6, 0.99, 0.999], [15, 17, 31, 64, 65, 12]), (2, 160, 16, 160, [0.99, 0.8], [1] * 9),
    (1, 500, 40, 20, [0.97], [1, 1]), (2, 7, 5, 6, [0.9, 0.5], [1] * 6)])
def test_retention_alone(device, dtype, H, dk, dv, dims, decay, lengths):
    """Segments that end before, at and behind a chunk's edge, far from the sequence's start, from a memory that is not
    zero, decays from zero to one; the outputs and, much sharper, the memory that is left, against float64.  The turned
    keys enter the memory as float32 numbers in either run dtype."""
    g = torch.Generator().manual_seed(H * 100 + dk + dv)
    N = sum(lengths)
    rnd = lambda *sh: torch.randn(*sh, generator=g)
    rows = rnd(N, 2 * H * (dk + dv)).to(dtype)
    bounds, slots, phase, pos, ctx = _step_arrays(lengths, 2, device, g, [17 * i + (900 if i % 2 else 0) for i in range(len(lengths))])
    state = rnd(len(lengths) + 2, 2, H, dv, dk)
    rot = None if dims is None else {"base": 10000.0, "dims": dims}
    want, left = _retained(rows, H, dk, dv, rot, decay, 1e-5, pos, state[slots, phase], bounds)
    st = state.clone().to(device)
    got = _ops(device).retention(rows.to(device), H, dk, dv, _rotation(rot, dk, device), _decays(decay, device), 1e-5, st, ctx)
    tol = 1e-2 if dtype == torch.bfloat16 else 5e-4
    assert got.dtype == dtype and torch.allclose(got.cpu().double(), want, rtol=tol, atol=tol), (got.cpu().double() - want).abs().max()
    _left_behind(st, state, slots, phase, left, 3e-5)


@pytest.mark.gpu
@pytest.mark.parametrize("dk,dv", [(64, 64), (128, 64), (256, 128), (48, 80)])
def test_retention_in_chunks_reads_queries_keys_and_memory_precisely(dk, dv):
    """bfloat16 rows: nearly all outputs in chunks are the rounding of the float64 numbers themselves (no turned query or
    key, weighted score or memory is read as one bfloat16 number)."""
    H, T = 2, 200
    g = torch.Generator().manual_seed(dk)
    rows = torch.randn(T, 2 * H * (dk + dv), generator=g).bfloat16()
    rows[:, 2 * H * dk + H * dv:] = 1.0
    front = torch.randn(1, H, dv, dk, generator=g)
    rot, decay = {"base": 1000.0, "dims": dk}, [0.97, 0.999]
    _, _, _, pos, ctx = _step_arrays([T], 0, "cuda:0", g)
    ctx.state_slots.zero_()
    ctx.state_phase.zero_()
    want, _ = _retained(rows, H, dk, dv, rot, decay, 1e-6, pos, front, [(0, T)])
    state = torch.zeros(1, 2, H, dv, dk)
    state[0, 0] = front[0]
    got = _ops("cuda:0").retention(rows.cuda(), H, dk, dv, _rotation(rot, dk, "cuda:0"), _decays(decay, "cuda:0"), 1e-6,
                                   state.cuda(), ctx)
    exact = got.cpu() == want.float().bfloat16()
    assert exact.float().mean() > 0.97, exact.float().mean()


# ---------------------------------------------------------------------------------------------- mixers over the cache
def _mixer_alone(folder, device, layer, sizes, x, dtype="float32", page_size=16, change=None):
    """Runs one layer's mixer over the paged cache and its per-request state in the given portions."""
    model = _load(folder, dtype, device)
    ops = _ops(device)
    mixer = model.blocks[layer].mixer
    if change is not None:
        change(mixer)
        mixer.finalize()
    pages = -(-sum(sizes) // page_size) + 1
    cache = CacheManager({0: mixer.cache_need()}, page_size=page_size, num_pages=pages, max_requests=1, dtype=model.dtype,
                         device=device, poison=True)
    outs, o = [], 0
    for n in sizes:
        if not cache.has_request("r"):
            cache.add_request("r")
        cache.reserve("r", n)
        ctx = build_context(ops, model.dtype, device, cache, [StepEntry("r", [0] * n, [])], model.config.vocab)
        gctx = ctx.groups[0]
        view = CacheView(0, True, kv=cache.groups[0].tensors.get(0), block_table=gctx.block_table,
                         slot_mapping=gctx.slot_mapping, attn_meta=gctx, group=0, pages=cache.groups[0].pages[0],
                         states=cache.named_state.get(0))
        y = mixer.forward(x[o:o + n].to(device).to(model.dtype), ctx, view)
        outs.append(ops.materialize(y).float().cpu())
        cache.commit("r")
        o += n
    return torch.cat(outs)


def _plain_mixer(cfg, w, layer, x, change=None):
    wd = _doubles(w)
    if change is not None:
        change(wd, f"l{layer}.mix.")
    lc = cfg["layers"][layer]
    return P.mixer(lc["type"], x.double(), wd, f"l{layer}.mix.", lc["mixer"], cfg["norm"]["eps"],
                   list(range(x.shape[0]))).float()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name,layer", [(n, i) for n in LIFESUN for i in range(len(LIFESUN[n]["layers"]))])
def test_mixers_alone(folders, device, name, layer):
    """Each pair of mixers whole, in portions down to two tokens and token by token (also the first tokens of a sequence
    one by one: shorter than the convolution's taps) equals the plain pair."""
    cfg, w = P.load(folders[name])
    T = 75
    x = torch.randn(T, cfg["width"], generator=torch.Generator().manual_seed(layer + 1))
    want = _plain_mixer(cfg, w, layer, x)
    for sizes in ([T], [30, 2, 17, 1, 1, 24], [1] * T):
        got = _mixer_alone(folders[name], device, layer, sizes, x)
        assert torch.allclose(got, want, rtol=3e-4, atol=3e-5), (sizes[:3], (got - want).abs().max())


@pytest.mark.gpu
@pytest.mark.parametrize("name,layer", [(n, i) for n in LIFESUN_FAST for i in range(len(LIFESUN_FAST[n]["layers"]))]
                         + [("LA", 0), ("LA", 1), ("LB", 0), ("LB", 1), ("LB", 3)])
def test_mixers_alone_in_bfloat16(folders_bf16, name, layer):
    cfg, w = P.load(folders_bf16[name])
    T = 310
    x = torch.randn(T, cfg["width"], generator=torch.Generator().manual_seed(layer + 1)).bfloat16().float()
    want = _plain_mixer(cfg, w, layer, x)
    for sizes in ([T], [63, 2, 64, 1, 16, 164], [129] + [1] * 181):
        got = _mixer_alone(folders_bf16[name], "cuda:0", layer, sizes, x, dtype="bfloat16")
        err = (got - want).abs().max() / want.abs().max()
        assert err < 2e-2, (sizes[:3], err)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("layer", [0, 1, 2])
def test_memory_long_decoding_through_both_halves_of_its_state(folders, device, layer):
    """Hundreds of single tokens; inputs large enough that decays and gates reach both their ends."""
    cfg, w = P.load(folders["LA"])
    T = 300
    x = torch.randn(T, cfg["width"], generator=torch.Generator().manual_seed(3)) * 2.0
    want = _plain_mixer(cfg, w, layer, x)
    for sizes in ([T], [3] + [1] * (T - 3), [149, 2, 149]):
        got = _mixer_alone(folders["LA"], device, layer, sizes, x)
        assert torch.allclose(got, want, rtol=5e-4, atol=5e-5), (got - want).abs().max()


# ---------------------------------------------------------------------------------------------- keys far away, edges
def _sharpen(mixer):
    """The attention's keys are projected with its first query heads' matrix, and norm weights are one: a token that has
    the direction of the last one then takes the last query's weight, if the query may see it.  Nothing turns, and the
    recurrent mixer beside it is silenced."""
    a = mixer.left
    nq, nk = a.num_heads * a.head_dim, a.num_kv_heads * a.head_dim
    rows, step = a.params["wqkv"], a.head_dim * (a.num_heads // a.num_kv_heads)
    for g in range(a.num_kv_heads):
        rows[nq + g * a.head_dim: nq + (g + 1) * a.head_dim].copy_(rows[g * step: g * step + a.head_dim])
    for name in ("q_norm", "k_norm"):
        if name in a.params:
            a.params[name].fill_(1.0)
    rot = a.position.rotation()
    if rot is not None:
        rot.inv_freq.zero_()
        a.position.rotation = lambda: rot
    mixer.right.params["wo"].zero_()


def _sharpen_plain(cfg, layer):
    m = cfg["layers"][layer]["mixer"]["left"]
    step = m["dim"] * (m["heads"] // m["kv_heads"])

    def change(wd, p):
        q = wd[p + "left.q"]
        wd[p + "left.k"] = torch.cat([q[g * step: g * step + m["dim"]] for g in range(m["kv_heads"])])
        for name in ("q.norm", "k.norm"):
            if p + "left." + name in wd:
                wd[p + "left." + name] = torch.ones_like(wd[p + "left." + name])
        wd[p + "right.o"] = torch.zeros_like(wd[p + "right.o"])

    return change


def _edge_case(folder, layer, T, special, big, device, sizes, dtype, tol, monkeypatch):
    cfg, w = P.load(folder)
    change = _sharpen_plain(cfg, layer)
    monkeypatch.setattr(P, "turn", lambda x, positions, rot: x)  # (angles of zero on both sides)
    x = torch.randn(T, cfg["width"], generator=torch.Generator().manual_seed(9))
    if dtype == "bfloat16":
        x = x.bfloat16().float()
    x[special] = big * x[T - 1]
    want = _plain_mixer(cfg, w, layer, x, change=change)
    got = _mixer_alone(folder, device, layer, sizes, x, dtype=dtype, change=_sharpen)
    assert (got - want).abs().max() < tol * want.abs().max(), (got - want).abs().max() / want.abs().max()
    x2 = x.clone()
    x2[special] = torch.randn(cfg["width"], generator=torch.Generator().manual_seed(1))
    return (_plain_mixer(cfg, w, layer, x2, change=change)[T - 1] - want[T - 1]).abs().max() / want[T - 1].abs().max()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("decoding", [False, True])
@pytest.mark.parametrize("layer,back", [(0, "chunk_first"), (0, "before_chunk"), (0, "start"), (0, "page_edge"),
                                        (1, "just_inside"), (1, "just_outside"), (1, "start"), (1, "page_edge")])
def test_one_key_that_stands_out_at_the_edges(folders, device, decoding, layer, back, monkeypatch):
    """One early token is given the last token's direction.  Just inside the chunk or window the last query's weight lies
    on it; just outside, or at the sequence's start, the query does not see it: the plain mixer says which, and the
    engine follows it, in a prompt and in decoding, hundreds of tokens on (chunks and windows of 48, pages of 16)."""
    T = 279 if layer == 0 else 290  # (the last query in the middle of the sixth chunk: positions 240 .. 287)
    special = {"chunk_first": 240, "before_chunk": 239, "start": 0, "page_edge": 255, "just_outside": T - 1 - 48,
               "just_inside": T - 48}[back]
    sizes = [special + 3] + [1] * (T - special - 3) if decoding else [T]
    moved = _edge_case(folders["LS"], layer, T, special, 3.0, device, sizes, "float32", 5e-4, monkeypatch)
    assert (moved > 1e-2) == (back not in ("before_chunk", "start", "just_outside")), moved


@pytest.mark.gpu
@pytest.mark.parametrize("decoding", [False, True])
@pytest.mark.parametrize("name,layer,size", [("LF", 0, 80), ("LF", 1, 112), ("LF", 2, 70), ("LF", 3, 100), ("LF", 4, 130),
                                             ("LW", 0, 90), ("LW", 1, 75)])
@pytest.mark.parametrize("outside", [False, True])
def test_one_key_that_stands_out_on_the_matrix_core_kernels(folders_bf16, decoding, name, layer, size, outside, monkeypatch):
    """The same in bfloat16 at head sizes that the matrix-core attention kernels take (capped scores, zero sinks)."""
    kind = lifesun_config_json(name)["layers"][layer]["type"]
    T = size * 3 + size // 2
    first = size * 3 if kind == "parallel" else T - size
    special = first - 1 if outside else first
    sizes = [special + 3] + [1] * (T - special - 3) if decoding else [T]
    moved = _edge_case(folders_bf16[name], layer, T, special, 2.0, "cuda:0", sizes, "bfloat16", 2e-2, monkeypatch)
    assert (moved > 5e-2) == (not outside), moved


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("decoding", [False, True])
def test_sink_of_zero_and_gates_per_head(folders, device, decoding):
    """A query alone in its chunk: without the sink its weight would be one whatever the score.  The gates tell the heads
    apart: taken from another head they would change the output by far more than the tolerance."""
    name, layer, T = "LA", 3, 121  # (chunks of 40: the last query is the first of its chunk)
    cfg, w = P.load(folders[name])
    x = torch.randn(T, cfg["width"], generator=torch.Generator().manual_seed(11))
    want = _plain_mixer(cfg, w, layer, x)
    got = _mixer_alone(folders[name], device, layer, [40] + [1] * (T - 40) if decoding else [T], x)
    assert torch.allclose(got, want, rtol=3e-4, atol=3e-5), (got - want).abs().max()
    flip = lambda wd, p: wd.update({p + "left.g": wd[p + "left.g"].flip(0)})
    assert (_plain_mixer(cfg, w, layer, x, change=flip) - want).abs().max() > 1e-2
    lc = cfg["layers"][layer]
    wd = _doubles(w)
    real = P.sink_softmax
    try:
        P.sink_softmax = lambda s, mask: torch.softmax(s.masked_fill(~mask, float("-inf")), dim=-1)
        plain = P.mixer(lc["type"], x.double(), wd, f"l{layer}.mix.", lc["mixer"], cfg["norm"]["eps"], list(range(T))).float()
    finally:
        P.sink_softmax = real
    assert (plain[T - 1] - want[T - 1]).abs().max() > 1e-2


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("decoding", [False, True])
def test_capped_scores_far_beyond_the_cap(folders, device, decoding):
    """Norm weights so large that scores run to many times the cap on both sides."""
    name, layer, T = "LA", 1, 90
    cfg, w = P.load(folders[name])
    x = torch.randn(T, cfg["width"], generator=torch.Generator().manual_seed(12))
    change = lambda mixer: mixer.left.params["q_norm"].mul_(40.0)
    change_plain = lambda wd, p: wd.update({p + "left.q.norm": wd[p + "left.q.norm"] * 40.0})
    want = _plain_mixer(cfg, w, layer, x, change=change_plain)
    got = _mixer_alone(folders[name], device, layer, [40] + [1] * (T - 40) if decoding else [T], x, change=change)
    assert torch.allclose(got, want, rtol=5e-4, atol=1e-4), (got - want).abs().max()
    cfg["layers"][layer]["mixer"]["left"]["softcap"] = 1e6
    assert (_plain_mixer(cfg, w, layer, x, change=change_plain) - want).abs().max() > 1e-1


@pytest.mark.gpu
@pytest.mark.parametrize("name,layer", [("LF", 0), ("LF", 3), ("LW", 1)])
def test_capped_scores_far_beyond_the_cap_on_the_matrix_core_kernels(folders_bf16, name, layer):
    """The same at every matrix-core head size, in prompts and in decoding.  (The scores' products are formed from
    queries and keys in bfloat16: beyond the cap their error is squashed with them.)"""
    cfg, w = P.load(folders_bf16[name])
    T = 170
    x = torch.randn(T, cfg["width"], generator=torch.Generator().manual_seed(12)).bfloat16().float()
    change = lambda mixer: mixer.left.params["q_norm"].mul_(8.0)
    change_plain = lambda wd, p: wd.update({p + "left.q.norm": wd[p + "left.q.norm"] * 8.0})
    want = _plain_mixer(cfg, w, layer, x, change=change_plain)
    for sizes in ([T], [100] + [1] * 70):
        got = _mixer_alone(folders_bf16[name], "cuda:0", layer, sizes, x, dtype="bfloat16", change=change)
        assert (got - want).abs().max() < 8e-2 * want.abs().max(), (got - want).abs().max() / want.abs().max()


# ---------------------------------------------------------------------------------------------- whole models
_PLAIN = {}


def _plain_logits(folder, toks):
    key = (folder, tuple(toks))
    if key not in _PLAIN:
        cfg, w = P.load(folder)
        _PLAIN[key] = P.forward(cfg, w, toks).float()
    return _PLAIN[key]


def _sensitivity(folder, toks):
    """Per position, the most that weights off by up to 2^-8 change the plain model's logits (of the largest logit)."""
    cfg, w = P.load(folder)
    ref, worst = _plain_logits(folder, toks).double(), None
    for draw in range(4):
        g = torch.Generator().manual_seed(draw)
        noisy = {k: v.double() * (1.0 + (2.0 * torch.rand(v.shape, generator=g, dtype=torch.float64) - 1.0) * 2.0 ** -8)
                 for k, v in w.items()}
        e = (P.forward(cfg, noisy, toks) - ref).abs().max(dim=-1).values / ref.abs().max()
        worst = e if worst is None else torch.maximum(worst, e)
    return worst


def _over(got, ref, folder, toks, dtype):
    """The positions whose error is over the tolerance, and all errors."""
    err = (got - ref).abs().max(dim=-1).values / ref.abs().max()
    over = err > TOL[dtype]
    if dtype == "bfloat16" and bool(over.any()):
        over &= err > 3.0 * _sensitivity(folder, toks)
    return over.nonzero().squeeze(-1).tolist(), err


def _check(name, folder, dtype, device, mode, record=False, page_size=16, lengths=None, top=None, seed=5):
    lengths = lengths or (LENGTHS[name] + (LENGTHS[name][::-1] if mode == "mixed" else []))
    vocab = (top or lifesun_config_json(name))["vocab"]
    reqs = traces.random_requests(vocab, lengths, seed=seed)
    steps = MODES[mode](reqs)
    runner = make_runner(folder, dtype, traces.max_live_tokens(steps), device, reference_ops=(device == "cpu"),
                         poison=True, max_requests=4, page_size=page_size, decode_graphs=None if record else False)
    handed = [collections.Counter() for _ in runner.cache.groups]
    for g, seen in zip(runner.cache.groups, handed):
        def alloc(n, inner=g.pool.alloc, seen=seen):
            pages = inner(n)
            seen.update(pages)
            return pages
        g.pool.alloc = alloc
    got = traces.run_trace(runner, steps)
    if record:
        assert runner.graphs is not None and runner.graphs.replays > 0
    if mode == "mixed" and top is None:  # pages and slots were used again
        assert all(max(seen.values()) > 1 for seen in handed)
        assert len(reqs) > runner.cache.max_requests
    runner.cache.check()
    assert runner.cache.num_live() == 0 and all(g.pool.num_held == 0 for g in runner.cache.groups)
    for rid, toks in reqs.items():
        ref = _plain_logits(folder, toks)
        assert got[rid].shape == ref.shape and torch.isfinite(got[rid]).all(), f"{rid}: non-finite logits"
        bad, err = _over(got[rid], ref, folder, toks, dtype)
        assert not bad, f"{name} {dtype} {mode} {rid}: first wrong position {bad[0]} of {len(toks)}, error {err[bad[0]]:.3g}"


@pytest.mark.parametrize("mode", list(MODES))
@pytest.mark.parametrize("name", list(LIFESUN))
def test_cpu_plain_ops_float32(folders, name, mode):
    _check(name, folders[name], "float32", "cpu", mode)


@pytest.mark.parametrize("page_size", [4, 64])
def test_cpu_other_page_sizes(folders, page_size):
    _check("LA", folders["LA"], "float32", "cpu", "mixed", page_size=page_size)


@pytest.mark.gpu
@pytest.mark.parametrize("mode", list(MODES))
@pytest.mark.parametrize("name", list(LIFESUN))
def test_gpu_float32(folders, name, mode):
    _check(name, folders[name], "float32", "cuda:0", mode)


@pytest.mark.gpu
@pytest.mark.parametrize("mode", ["tail", "mixed"])
@pytest.mark.parametrize("name", list(LIFESUN))
def test_gpu_float32_with_recorded_decode_steps(folders, name, mode):
    _check(name, folders[name], "float32", "cuda:0", mode, record=True)


@pytest.mark.gpu
@pytest.mark.parametrize("mode", list(MODES))
@pytest.mark.parametrize("name", list(LIFESUN) + list(LIFESUN_FAST))
def test_gpu_bfloat16(folders_bf16, name, mode):
    _check(name, folders_bf16[name], "bfloat16", "cuda:0", mode)


@pytest.mark.gpu
@pytest.mark.parametrize("page_size", [4, 64])
def test_gpu_other_page_sizes(folders, page_size):
    _check("LA", folders["LA"], "float32", "cuda:0", "mixed", page_size=page_size)


@pytest.mark.gpu
@pytest.mark.parametrize("name", ["LA", "LB", "LF", "LW"])
def test_gpu_bfloat16_recorded_decode_steps_equal_unrecorded_ones(folders_bf16, name):
    """Steps of single tokens replayed from recorded graphs give the bits of the same steps run launch by launch:
    the memories' two halves, the convolutions' rows, the angles and the pages are those of the step, not of the
    recording."""
    reqs = traces.random_requests(lifesun_config_json(name)["vocab"], [90, 41, 67], seed=6)
    steps = traces.tail(reqs, last=40)
    outs = []
    for graphs in (None, False):
        runner = make_runner(folders_bf16[name], "bfloat16", traces.max_live_tokens(steps), "cuda:0", poison=True,
                             max_requests=4, decode_graphs=graphs)
        outs.append(traces.run_trace(runner, steps))
        if graphs is None:
            assert runner.graphs is not None and runner.graphs.replays > 0
    for rid in reqs:
        assert torch.equal(outs[0][rid], outs[1][rid])


@pytest.mark.gpu
@pytest.mark.parametrize("name", list(LIFESUN_FAST))
def test_gpu_float32_at_vector_sizes(tmp_path, name):
    folder = write_lifesun(name, str(tmp_path / name), torch.float32)
    for mode in ("whole", "portions", "mixed"):
        _check(name, folder, "float32", "cuda:0", mode)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", list(range(16)))
def test_gpu_configurations_drawn_at_random(tmp_path, seed, dtype):
    from jax_llm_examples_amd.weights import write_random_model

    top, page_size, lengths = draw_lifesun(seed)
    arch = get_architecture("Lifesun")
    folder = write_random_model(arch, arch.parse_config(top), str(tmp_path / "m"), seed,
                                torch.float32 if dtype == "float32" else torch.bfloat16)
    _check("drawn", folder, dtype, "cuda:0", "mixed", page_size=page_size, lengths=lengths, top=top, seed=seed)


@pytest.mark.parametrize("seed", [0, 1, 2])
def test_cpu_configurations_drawn_at_random(tmp_path, seed):
    from jax_llm_examples_amd.weights import write_random_model

    top, page_size, lengths = draw_lifesun(seed)
    arch = get_architecture("Lifesun")
    folder = write_random_model(arch, arch.parse_config(top), str(tmp_path / "m"), seed, torch.float32)
    _check("drawn", folder, "float32", "cpu", "mixed", page_size=page_size, lengths=lengths, top=top, seed=seed)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", ["LA", "LB"])
def test_residual_stream_behind_every_layer_run(folders, device, name):
    """What a watcher of the step sees behind every run of a layer equals the plain model's stream."""
    folder = folders[name]
    cfg, w = P.load(folder)
    toks = traces.random_requests(128, [29], seed=2)["r0"]
    want = []
    P.forward(cfg, w, toks, taps=want)
    runner = make_runner(folder, "float32", 64, device, reference_ops=(device == "cpu"), max_requests=2)
    seen = []
    runner.step([StepEntry("r", toks, [])], tap=lambda part_, nm, value: seen.append(value()) if nm == "residual" else None)
    assert len(seen) == len(want) == len(P.run_order(cfg))
    for a, b in zip(seen, want):
        assert torch.allclose(a.cpu(), b.float(), rtol=1e-4, atol=1e-4)


def test_every_run_of_a_looped_layer_has_a_cache_and_state_of_its_own(folders):
    model = _load(folders["LA"], "float32", "cpu")
    assert [e.layer for e in model.plan.order] == [0, 1, 2, 1, 2, 1, 2, 3]
    assert [e.enters_pass for e in model.plan.order] == [None, 0, None, 1, None, 2, None, None]
    assert len({e.cache for e in model.plan.order}) == 8 and all(e.writes_cache for e in model.plan.order)


@pytest.mark.parametrize("device", DEVICES)
def test_a_batch_gives_what_each_request_alone_gives(folders, device):
    """One step with prompts of unequal length, portions and single tokens beside each other against every request on
    its own."""
    reqs = traces.random_requests(300, [61, 1, 18, 40], seed=8)
    alone = {}
    for rid, toks in reqs.items():
        runner = make_runner(folders["LA"], "float32", 128, device, reference_ops=(device == "cpu"), max_requests=4)
        alone[rid] = runner.step([StepEntry(rid, toks, list(range(len(toks))))]).float().cpu().clone()
    runner = make_runner(folders["LA"], "float32", 256, device, reference_ops=(device == "cpu"), max_requests=4, poison=True)
    at = {rid: 0 for rid in reqs}
    got = {rid: [] for rid in reqs}
    for cut in ((20, 1, 2, 39), (1, 0, 1, 1), (40, 0, 15, 0)):
        entries = [StepEntry(rid, toks[at[rid]: at[rid] + n], list(range(n)))
                   for (rid, toks), n in zip(reqs.items(), cut) if n]
        logits = runner.step(entries).float().cpu().clone()
        o = 0
        for e in entries:
            got[e.rid].append(logits[o: o + len(e.tokens)])
            o += len(e.tokens)
            at[e.rid] += len(e.tokens)
    for rid in reqs:
        assert torch.allclose(torch.cat(got[rid]), alone[rid], rtol=1e-4, atol=1e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["parallel", "parallel_2"])
def test_a_token_far_back_matters_through_the_memory_alone(device, tmp_path, kind):
    """Every window and chunk ends long before it: the logits at the last token still change with a token 130 places
    back, through the recurrent memory (whose decay is made slow); the engine follows the plain model in a prompt and
    in decoding."""
    from safetensors.torch import save_file

    from jax_llm_examples_amd.weights import write_random_model

    top = lifesun_config_json("LA")
    top["layers"] = [json.loads(json.dumps(lc)) for lc in top["layers"] if lc["type"] == kind][:1]
    del top["loop"]
    right = top["layers"][0]["mixer"]["right"]
    if kind == "parallel_2":
        right["decay"] = [0.999] * right["heads"]
    arch = get_architecture("Lifesun")
    folder = write_random_model(arch, arch.parse_config(top), str(tmp_path / "slow"), 2, torch.float32)
    if kind == "parallel":
        _, w = P.load(folder)
        w["l0.mix.right.lam"] = torch.full_like(w["l0.mix.right.lam"], -9.0)
        save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(folder, "model.safetensors"))
    toks = traces.random_requests(300, [160], seed=4)["r0"]
    i = 159

    def logits_at(seq, decoding):
        runner = make_runner(folder, "float32", 256, device, reference_ops=(device == "cpu"), max_requests=2)
        if not decoding:
            runner.step([StepEntry("r", seq[:i], [])])
        else:
            runner.step([StepEntry("r", seq[:130], [])])
            for t in range(130, i):
                runner.step([StepEntry("r", [seq[t]], [])])
        return runner.step([StepEntry("r", [seq[i]], [0])])[0].cpu().clone()

    other = list(toks)
    other[29] = (toks[29] + 1) % 300
    for decoding in (False, True):
        a, b = logits_at(toks, decoding), logits_at(other, decoding)
        wa, wb = _plain_logits(folder, toks)[i], _plain_logits(folder, other)[i]
        assert (wa - wb).abs().max() > 1e-3
        assert torch.allclose(a, wa, rtol=5e-5, atol=5e-5) and torch.allclose(b, wb, rtol=5e-5, atol=5e-5)


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_engine(folders, device):
    """``Engine.generate`` with its scheduler (portions of prompts beside decoded tokens, four requests at a time)
    gives the plain model's greedy tokens."""
    name = "LA"
    g = torch.Generator().manual_seed(1)
    prompts = [torch.randint(0, 300, (n,), generator=g).tolist() for n in (7, 40, 19, 3, 55)]
    steps = 10
    want = []
    for p in prompts:
        seq = list(p)
        for _ in range(steps):
            seq.append(int(_plain_logits(folders[name], seq)[-1].argmax()))
        want.append(seq[len(p):])
    engine = Engine(_load(folders[name], "float32", device), cache_tokens=512, decode_batch_size=4,
                    max_num_batched_tokens=24, **({"reference_ops": True} if device == "cpu" else {}))
    assert engine.generate(prompts, SamplingParams(max_decode_length=steps)) == want


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run_program(folders_bf16, tmp_path, dtype):
    """``bin/trace_run`` as a program, on a folder that holds config.json and bfloat16 weights."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    folder = folders_bf16["LA"]
    reqs = traces.random_requests(300, [40, 9, 70, 21, 33], seed=11)
    steps = traces.mixed(reqs)
    out_dir = tmp_path / "out"
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", dtype,
                           "--out", str(out_dir), "--max-tokens", str(traces.max_live_tokens(steps)),
                           "--max-requests", "4"],
                          input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [ln for ln in proc.stdout.splitlines() if ln.startswith("done")] == [f"done {s['step']}" for s in steps]
    rows = {rid: [] for rid in reqs}
    for s in steps:
        got = torch.from_numpy(np.fromfile(out_dir / f"{s['step']}.f32", dtype="<f4").reshape(-1, 300))
        o = 0
        for e in s["entries"]:
            rows[e["id"]].append(got[o: o + len(e["want"])])
            o += len(e["want"])
    for rid, toks in reqs.items():
        bad, err = _over(torch.cat(rows[rid]), _plain_logits(folder, toks), folder, toks, dtype)
        assert not bad, (rid, bad[0], err[bad[0]])


# ---------------------------------------------------------------------------------------------- configuration
def test_configuration_round_trip_and_errors():
    arch = get_architecture("Lifesun")
    for name in list(LIFESUN) + list(LIFESUN_FAST):
        top = lifesun_config_json(name)
        cfg = arch.parse_config(top)
        assert arch.parse_config(arch.config_to_dict(cfg)) == cfg
        assert len(arch.plan(cfg).layers) == len(top["layers"])
    for seed in range(30):
        top, _, _ = draw_lifesun(seed)
        cfg = arch.parse_config(top)
        assert arch.parse_config(arch.config_to_dict(cfg)) == cfg

    def refused(*path_and_value):
        *path, key, value = path_and_value
        bad = json.loads(json.dumps(lifesun_config_json("LA")))
        d = bad
        for k in path:
            d = d[k]
        d[key] = value
        with pytest.raises(ConfigError):
            arch.parse_config(bad)

    mix = lambda i, side: ("layers", i, "mixer", side)
    refused(*mix(0, "left"), "kv_heads", 3)  # (four heads on three kv heads)
    refused(*mix(0, "left"), "softcap", 5.0)  # (a key this mixer does not have)
    refused(*mix(0, "left"), "mask", {"size": 0})
    refused(*mix(1, "left"), "softcap", 0.0)
    refused(*mix(1, "left"), "rot", {"base": 10.0, "dims": 18})  # (more than the head has)
    refused(*mix(0, "right"), "blocks", 5)  # (48 channels in five blocks)
    refused(*mix(1, "right"), "decay", [0.5, 0.9])  # (three heads)
    refused(*mix(1, "right"), "decay", [0.5, 0.9, 1.5])
    refused("layers", 0, "type", "parallel_3")
    refused("layers", 0, "mlp", {"kind": "moe", "ff": 4})
    refused("loop", {"start": 1, "stop": 9, "times": 2})
    refused("loop", {"start": 2, "stop": 2, "times": 2})
    refused("logit_softcap", 3.0)


def test_missing_and_misshapen_tensors(folders, tmp_path):
    """A checkpoint that lacks a tensor or gives one another shape is refused by name."""
    from safetensors.torch import save_file

    from jax_llm_examples_amd.weights.loader import WeightsError

    cfg, w = P.load(folders["LA"])
    w["l0.mix.right.ra"] = w["l0.mix.right.ra"].reshape(48, 16)
    del w["l1.mix.left.q.norm"]
    (tmp_path / "bad").mkdir()
    with open(tmp_path / "bad" / "config.json", "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "bad" / "model.safetensors"))
    with pytest.raises(WeightsError) as e:
        _load(str(tmp_path / "bad"), "float32", "cpu")
    assert "l1.mix.left.q.norm" in str(e.value) and "l0.mix.right.ra" in str(e.value)
