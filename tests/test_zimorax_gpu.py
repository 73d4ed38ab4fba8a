"""Zimorax on the GPU against the plain implementation (plain_zimorax.py): every mechanism alone, then the engine
whole / token by token / in portions / in ragged batches with reused slots / through graphs and the generation loop,
in float32 and bfloat16, at sizes that differ from one another in everything.

bfloat16 is judged like the other models of this folder: the plain implementation run with bfloat16 storage, and with
random errors of that size in its place, shows what that type costs at every position, and the engine may be a small
multiple of that off.  Norms over a head's few entries make single positions ill-conditioned now and then (a draw of
rounding errors in ten moves one by ten times the usual), so one position in fifty may be further off; a wrong key or state
shows in float32, where every position counts, and in the kernels' own tests.  Mistakes that a comparison must
notice are planted in the plain implementation."""

import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

pytestmark = pytest.mark.gpu

import plain_zimorax as P  # noqa: E402
from gpu_checks import Expected  # noqa: E402

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEV = "cuda"
DTYPES = ["float32", "bfloat16"]
BF16_MARGIN = 3.0
BF16_FURTHER_OFF = 0.02
DRAWS = 4


def talking(heads, kv, dim, vdim, size, rot_dims, base=10000.0, factor=2.0, original=64, fast=8.0, slow=1.0, scale=0.2):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "mask": {"size": size}, "scale": scale,
                                           "rot": {"base": base, "dims": rot_dims,
                                                   "scaling": {"factor": factor, "original": original, "fast": fast, "slow": slow}}}}


def mamba(heads, vdim, state, groups, conv=4, norm_groups=1):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}}


def delta(heads, kv, dim, vdim, conv=4):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}}


def layer(mixer, ff):
    return dict(mixer, mlp={"kind": "dense", "ff": ff} if ff else None)


CONFIGS = {
    # values of another size than keys, grouped heads everywhere, a part of every head rotated, convolutions of 2, 3 and 4
    # taps, a layer without a feed-forward, a loop of two passes in the middle that holds every kind of mixer
    "A": dict(vocab=300, width=128, norm={"eps": 1e-5}, loop={"start": 1, "stop": 4, "times": 2}, max_positions=1024, layers=[
        layer(mamba(4, 24, 16, 2, conv=3, norm_groups=2), 160),
        layer(delta(4, 2, 16, 24, conv=2), None),
        layer(talking(6, 3, 32, 24, 40, 16), 96),
        layer(mamba(3, 16, 40, 1, conv=4, norm_groups=3), 64),
        layer(delta(2, 2, 24, 16, conv=4), 48),
    ]),
    # sizes that are no multiples of 8 (rows that the matrix instructions cannot load); the loop is the whole model, three
    # passes; a window of five tokens; one kv head; a convolution of one tap; a state of 10 rows; as many groups as heads
    "B": dict(vocab=257, width=100, norm={"eps": 1e-6}, loop={"start": 0, "stop": 3, "times": 3}, max_positions=1024, layers=[
        layer(talking(3, 1, 20, 36, 5, 6, base=500.0, factor=8.0, original=30, fast=3.0, slow=0.5), 60),
        layer(mamba(3, 10, 10, 3, conv=1, norm_groups=5), 36),
        layer(delta(3, 1, 12, 20, conv=5), None),
    ]),
    # sizes at which bfloat16 runs the matrix-instruction kernels: four query heads a kv head, rows of 256 entries; a state
    # of 128 rows and channels of 64; a window that ends inside a page; the loop is one layer, twice
    "C": dict(vocab=512, width=256, norm={"eps": 1e-6}, loop={"start": 2, "stop": 3, "times": 2}, max_positions=2048, layers=[
        layer(mamba(8, 64, 128, 2, norm_groups=4), 384),
        layer(delta(8, 4, 32, 64), 256),
        layer(talking(8, 2, 128, 128, 100, 64, base=500000.0, original=512, fast=16.0, scale=0.09), 256),
        layer(mamba(4, 32, 64, 1), None),
    ]),
    # no loop; more than 16 heads, an odd number a kv head, rows above 512 entries with long values (the prompt kernel does
    # not take them); a window longer than any sequence; a factor of one (no stretching); a state of 200 rows
    "D": dict(vocab=400, width=192, norm={"eps": 1e-4}, loop=None, max_positions=1024, layers=[
        layer(talking(18, 6, 96, 96, 1000, 96, factor=1.0, scale=0.1), 128),
        layer(mamba(2, 72, 200, 1, conv=8, norm_groups=8), 96),
        layer(talking(10, 10, 40, 56, 33, 4, base=100.0, factor=16.0, original=20, fast=2.0, slow=0.1), 64),
    ]),
}


@pytest.fixture(scope="module")
def lib():
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    import fms_amd
    from fms_amd.kernels import load

    load()
    return fms_amd


def write_folder(lib, folder, cfg_kw, seed, sharp=1.0):
    """A model folder with random weights in which every learned number matters: norm weights and branch scales away from
    one, biases, mixing matrices away from the identity, slow and fast decays, step vectors of some size.
    sharp: a factor on the queries, so that single keys hold most of a query's weight."""
    from fms_amd.weights import write_safetensors

    lib.write_model_folder(folder, lib.ZimoraxConfig(**cfg_kw), seed=seed, architecture="zimorax", std=0.08)
    cfg, tensors = P.load_model_folder(folder)
    gen = torch.Generator().manual_seed(seed)

    def noise(t, std):
        return torch.randn(t.shape, generator=gen, dtype=torch.float64) * std

    for k in list(tensors):
        t = tensors[k]
        if k.endswith((".norm1", ".norm2", "final.norm", ".mix.norm")):
            tensors[k] = 1 + noise(t, 0.2)
        elif k.endswith((".ls1", ".ls2")):
            tensors[k] = 0.7 + noise(t, 0.2)
        elif k.endswith((".q.b", ".k.b", ".v.b", ".up.b", ".down.b", ".conv.b")):
            tensors[k] = noise(t, 0.3)
        elif k.endswith(".conv"):
            tensors[k] = noise(t, 0.5)
        elif k.endswith(".talk"):
            tensors[k] = torch.eye(t.shape[0], dtype=torch.float64) * 0.7 + noise(t, 0.4)
        elif k.endswith(".A_log"):
            tensors[k] = torch.rand(t.shape, generator=gen, dtype=torch.float64) * 5 - 3
        elif k.endswith(".dt_bias"):
            tensors[k] = noise(t, 1.0) - 1
        elif k.endswith(".mix.D"):
            tensors[k] = 1 + noise(t, 0.5)
        elif k == "loop.step":
            tensors[k] = noise(t, 0.5)
        elif k.endswith((".mix.in", "loop.in", "embed", "head")) or k.endswith((".mix.q", ".mix.k", ".mix.v")):
            tensors[k] = t * 2
    if sharp != 1.0:
        for i, entry in enumerate(cfg["layers"]):
            if entry["type"] == "attention":
                for n in ("q", "q.b"):
                    tensors[f"l{i}.mix.{n}"] = tensors[f"l{i}.mix.{n}"] * sharp
    tensors = {k: v.to(torch.bfloat16) for k, v in tensors.items()}
    write_safetensors(os.path.join(folder, "model.safetensors"), [(k, tuple(v.shape), v.dtype) for k, v in tensors.items()],
                      lambda name: tensors[name])
    return folder


@pytest.fixture(scope="module")
def folders(tmp_path_factory, lib):
    return {name: write_folder(lib, str(tmp_path_factory.mktemp(f"zimorax_{name}")), kw, 3 + i) for i, (name, kw) in enumerate(CONFIGS.items())}


_models, _plain, _expected = {}, {}, {}


def get(lib, folders, name, dtype):
    if (name, dtype) not in _models:
        _models[(name, dtype)] = lib.get_model("hf_pretrained", model_path=folders[name], data_type=dtype)
    return _models[(name, dtype)]


def plain(folders, name):
    if name not in _plain:
        _plain[name] = P.load_model_folder(folders[name])
    return _plain[name]


def tokens_for(vocab, n, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def expect(cfg, weights, ids, dtype) -> Expected:
    """Exact logits; for bfloat16 also the plain implementation's own error with bfloat16 storage at every position (the
    largest over several draws of rounding errors), and its 90th percentile over the sequence."""
    exact = P.forward(cfg, weights, ids).float()
    if dtype == "float32":
        return Expected(exact)
    error = torch.stack([(P.forward(cfg, weights, ids, rounding=r).float() - exact).abs().amax(dim=-1)
                         for r in ("bfloat16", *range(DRAWS))]).amax(dim=0)
    return Expected(exact, error, torch.quantile(error, 0.9).expand_as(error))


def expected_for(folders, name, n, seed, dtype):
    key = (name, n, seed, dtype)
    if key not in _expected:
        cfg, weights = plain(folders, name)
        ids = tokens_for(cfg["vocab"], n, seed)
        _expected[key] = (ids, expect(cfg, weights, ids, dtype))
    return _expected[key]


def judge(got, want, dtype):
    got = got.float().cpu()
    assert got.shape == want.shape, f"{tuple(got.shape)} logits, {tuple(want.shape)} expected"
    if dtype == "float32":
        torch.testing.assert_close(got, want.logits, atol=5e-4, rtol=1e-3)
        return
    error = (got - want.logits).abs().amax(dim=-1).flatten()
    ref, typical = want.ref_error.flatten(), want.typical.flatten()
    allowed = BF16_MARGIN * torch.maximum(ref, typical)
    worst = int(torch.argmax(error / allowed))
    assert bool(torch.isfinite(error).all())
    assert int((error > allowed).sum()) <= max(1, int(BF16_FURTHER_OFF * error.numel())), (
        f"{int((error > allowed).sum())} of {error.numel()} bfloat16 logits are far off, the worst "
        f"{float(error[worst]):.4g} off at row {worst}; the plain implementation with bfloat16 storage is "
        f"{float(ref[worst]):.4g} off there and typically {float(typical[worst]):.4g} (allowed: {BF16_MARGIN} times the larger)")
    if error.numel() >= 32:
        assert float(error.median()) <= float(ref.median()), (
            f"bfloat16 logits are {float(error.median()):.4g} off at the median, the plain implementation with bfloat16 storage {float(ref.median()):.4g}")


def i32(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


# ---- mechanisms alone ------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [100, 128, 257, 2048, 17000])
def test_layer_norm_with_a_scale_on_the_branch(lib, dtype, width):
    """stream += branch * scale; out = (stream - mean) / deviation * weight, also for chosen rows only (which must leave the
    stream alone), with a mean far from zero; and the stream as rows of the activation type in a wider buffer."""
    from fms_amd.kernels import ops

    gen = torch.Generator().manual_seed(width)
    T = 5
    x = torch.randn(T, width, generator=gen) + 30.0
    branch = torch.randn(T, width, generator=gen).to(dtype)
    scale, w = torch.randn(width, generator=gen), 1 + 0.3 * torch.randn(width, generator=gen)
    want_stream = x.double() + branch.double() * scale.double()
    want = P.layer_norm(want_stream, w.double(), 1e-3)
    tol = dict(atol=3e-5, rtol=1e-4) if dtype == torch.float32 else dict(atol=2e-2, rtol=1e-2)
    dev = [t.to(DEV) for t in (x, branch, scale, w)]
    resid = dev[0].clone()
    got = ops.add_norm(resid, dev[1], dev[3], None, 1e-3, dtype, use_mean=True, branch_scale=dev[2])
    torch.testing.assert_close(got.double().cpu(), want, **tol)
    torch.testing.assert_close(resid.double().cpu(), want_stream, atol=1e-5, rtol=1e-6)
    resid = dev[0].clone()
    got = ops.add_norm(resid, dev[1], dev[3], None, 1e-3, dtype, i32([3, 0]), True, dev[2])
    torch.testing.assert_close(got.double().cpu(), want[[3, 0]], **tol)
    assert torch.equal(resid, dev[0])
    wide = torch.zeros(T, 2 * width, dtype=dtype, device=DEV)
    ops.stream_rows(resid, dev[1], dev[2], wide[:, width:])
    torch.testing.assert_close(wide[:, width:].double().cpu(), want_stream, atol=1e-4 if dtype == torch.float32 else 0.3, rtol=1e-2)
    assert float(wide[:, :width].abs().max()) == 0 and torch.equal(resid, dev[0])
    ops.stream_rows(resid, None, None, wide[:, :width])
    assert torch.equal(wide[:, :width], dev[0].to(dtype))


def test_the_square_of_relu_and_a_convolution_with_silu(lib):
    from fms_amd.kernels import ops

    gen = torch.Generator().manual_seed(1)
    z = torch.randn(7, 33, generator=gen) * 3
    torch.testing.assert_close(ops.activation(z.to(DEV), "relu2").cpu(), torch.relu(z) ** 2)
    for C, taps, T in ((40, 4, 90), (27, 1, 70), (64, 2, 20), (36, 8, 200)):
        x = torch.randn(T, C + 9, generator=gen)
        w, b = torch.randn(C, taps, generator=gen) * 0.5, torch.randn(C, generator=gen)
        want = P.silu(P.causal_conv(x[:, 4 : 4 + C].double(), w.double(), b.double())).float()
        for cuts in ([T], [3, 2, T - 5], [T - 2, 1, 1], [1] * 12 + [T - 12]):
            state = torch.zeros(2, max(taps - 1, 1), C, device=DEV)
            got, at = [], 0
            for n in cuts:
                got.append(ops.short_conv(x[at : at + n].to(DEV), 4, C, w.to(DEV), b.to(DEV), state if taps > 1 else None, i32([0] * n), i32([1]),
                                          torch.float32, single_tokens=n == 1, activation="silu"))
                at += n
            torch.testing.assert_close(torch.cat(got).cpu(), want, atol=2e-5, rtol=1e-4)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,dim", [(1, 8), (3, 20), (4, 64), (2, 200), (20, 128)])
def test_values_normed_head_by_head(lib, dtype, heads, dim):
    from fms_amd.kernels import ops

    gen = torch.Generator().manual_seed(dim)
    proj = torch.randn(6, 17 + heads * dim + 3, generator=gen) * 0.01  # small: eps counts
    got = ops.value_head_norm(proj.to(DEV), 17, heads, dim, 1e-4, dtype, i32([0, 0, 1, 1, 1, 2]))
    values = P.over_rms(proj[:, 17 : 17 + heads * dim].double().view(6, heads, dim), 1e-4).view(6, -1)
    want = torch.cat([proj[:, :17].double(), values], dim=1)
    torch.testing.assert_close(got.double().cpu(), want, **(dict(atol=1e-6, rtol=1e-5) if dtype == torch.float32 else dict(atol=1e-4, rtol=1e-2)))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("cols,parts", [(48, 1), (96, 3), (50, 5), (4096, 8), (4096, 1), (20000, 2)])
def test_gated_norm_in_parts(lib, dtype, cols, parts):
    """The gate before the norm, each part over its own root mean square (one part far larger than the others)."""
    from fms_amd.kernels import ops

    gen = torch.Generator().manual_seed(cols + parts)
    y, rows = torch.randn(4, cols, generator=gen), torch.randn(4, cols + 10, generator=gen)
    y[:, : cols // parts] *= 50
    w = (1 + 0.3 * torch.randn(cols, generator=gen)).to(dtype)
    got = ops.gated_group_norm(y.to(DEV), rows.to(DEV)[:, :cols], w.to(DEV), parts, 1e-3, dtype, i32([0, 0, 1, 1]))
    want = P.gated_group_norm(y.double(), rows[:, :cols].double(), w.double(), parts, 1e-3)
    torch.testing.assert_close(got.double().cpu(), want, **(dict(atol=1e-5, rtol=1e-4) if dtype == torch.float32 else dict(atol=2e-2, rtol=1e-2)))


SSD_SIZES = [  # heads, vdim, groups, state
    (2, 16, 1, 16), (4, 24, 2, 40), (3, 10, 3, 10), (8, 64, 2, 128), (2, 72, 1, 200), (6, 8, 1, 1), (9, 33, 3, 64), (20, 16, 1, 256), (1, 1, 1, 7)]


def ssd_inputs(sizes, T, seed, a_range=(-3.0, 2.0)):
    H, Pd, G, N = sizes
    gen = torch.Generator().manual_seed(seed)
    xbc = torch.randn(T, H * Pd + 2 * G * N, generator=gen)
    dt = torch.randn(T, H + 3, generator=gen) - 1
    a_log = torch.rand(H, generator=gen) * (a_range[1] - a_range[0]) + a_range[0]
    return xbc, dt, a_log, torch.randn(H, generator=gen) * 0.5, torch.randn(H, generator=gen)


def ssd_want(sizes, xbc, dt, a_log, dt_bias, skip):
    H, Pd, G, N = sizes
    x, B, C = xbc.double().split([H * Pd, G * N, G * N], dim=1)
    T = xbc.shape[0]
    d = P.softplus(dt[:, :H].double() + dt_bias.double())
    return P.ssd_recurrence(x.reshape(T, H, Pd), B.reshape(T, G, N), C.reshape(T, G, N), d, a_log.double(), skip.double()).reshape(T, H * Pd)


def ssd_run(sizes, inputs, state, lens, slots, chunked, rows=None):
    from fms_amd.kernels import ops

    H, Pd, G, N = sizes
    xbc, dt, a_log, dt_bias, skip = [t.to(DEV) for t in inputs]
    starts = [0]
    for n in lens:
        starts.append(starts[-1] + n)
    seq = [b for b, n in enumerate(lens) for _ in range(n)]
    return ops.ssd(xbc, dt[:, :H], a_log, dt_bias, skip, state, i32(starts), i32(seq), i32(slots), len(lens), H, Pd, G, N, max(lens), chunked).cpu()


@pytest.mark.parametrize("sizes", SSD_SIZES)
def test_state_space_recurrence_whole_in_portions_and_in_a_batch(lib, sizes):
    """Token by token and in chunks, whole and in portions of any size, a ragged batch in slots that held other sequences:
    all against the plain recurrence."""
    H, Pd, G, N = sizes
    T = 150
    inputs = ssd_inputs(sizes, T, sum(sizes))
    want = ssd_want(sizes, *inputs)
    tol = dict(atol=2e-4, rtol=1e-4)
    for chunked, cuts in ((False, [T]), (True, [T]), (True, [64, 64, 22]), (True, [2, 65, 1, 63, 19]), (False, [1] * 20 + [130]),
                          (None, [100] + [1] * 5 + [2, 2, 41])):
        state = torch.zeros(3, H, Pd, N, device=DEV)
        got, at = [], 0
        for n in cuts:
            part = (inputs[0][at : at + n], inputs[1][at : at + n], *inputs[2:])
            got.append(ssd_run(sizes, part, state, [n], [1], chunked))
            at += n
        torch.testing.assert_close(torch.cat(got).double(), want, **tol)
        assert float(state[0].abs().max()) == 0 and float(state[2].abs().max()) == 0
    # a ragged batch: every sequence equals itself alone; the states end up where token by token leaves them
    lens = [70, 1, 64, 15]
    parts = [ssd_inputs(sizes, n, 40 + n) for n in lens]
    shared = parts[0][2:]
    parts = [(p[0], p[1], *shared) for p in parts]
    joined = (torch.cat([p[0] for p in parts]), torch.cat([p[1] for p in parts]), *shared)
    ends = []
    for chunked in (True, False):
        state = torch.full((6, H, Pd, N), 7.0, device=DEV)
        slots = [4, 0, 2, 5]
        state[slots] = 0
        got = ssd_run(sizes, joined, state, lens, slots, chunked).double()
        at = 0
        for p, n in zip(parts, lens):
            torch.testing.assert_close(got[at : at + n], ssd_want(sizes, *p), **tol)
            at += n
        assert float((state[[1, 3]] - 7).abs().max()) == 0
        ends.append(state.cpu())
    torch.testing.assert_close(ends[0], ends[1], **tol)


def test_state_space_recurrence_far_tokens_strong_decays_and_a_lost_state(lib):
    """A decay of 0.9999 a token carries the first token across 700; decays of hundreds of e-folds inside a chunk next to
    steps so small that their own decay is nothing must keep neighbours exact; a state lost between two steps shows."""
    sizes = (2, 16, 1, 32)
    H, Pd, G, N = sizes
    T = 700
    xbc, dt, a_log, dt_bias, skip = ssd_inputs(sizes, T, 5)
    far = xbc.clone()
    far[1:, : H * Pd] *= 1e-3
    far[0, : H * Pd] *= 30
    a_log = torch.full((H,), float(np.log(1e-4)))
    dt = torch.full_like(dt, float(np.log(np.expm1(1.0))))  # softplus gives 1
    args = (far, dt, a_log, torch.zeros(H), skip)
    want = ssd_want(sizes, *args)
    without = ssd_want(sizes, torch.cat([far[:1] * 0, far[1:]]), *args[1:])
    assert float((want - without)[-1].abs().max()) > 50 * float(without[-1].abs().max())  # the first token is what shows
    for chunked in (True, False):
        got = ssd_run(sizes, args, torch.zeros(1, H, Pd, N, device=DEV), [T], [0], chunked)
        torch.testing.assert_close(got.double(), want, atol=1e-3, rtol=1e-4)
    strong = torch.where(torch.arange(T)[:, None] % 5 == 0, torch.tensor(40.0), torch.tensor(-9.0)).expand(T, H + 3).contiguous()
    args = (xbc, strong, torch.full((H,), 2.0), torch.zeros(H), skip)
    want = ssd_want(sizes, *args)
    for chunked in (True, False):
        got = ssd_run(sizes, args, torch.zeros(1, H, Pd, N, device=DEV), [T], [0], chunked)
        torch.testing.assert_close(got.double(), want, atol=1e-3, rtol=2e-5)
    state = torch.zeros(1, H, Pd, N, device=DEV)
    inputs = ssd_inputs(sizes, T, 6, a_range=(-6.0, -4.0))
    want = ssd_want(sizes, *inputs)
    ssd_run(sizes, (inputs[0][:600], inputs[1][:600], *inputs[2:]), state, [600], [0], None)
    kept = ssd_run(sizes, (inputs[0][600:], inputs[1][600:], *inputs[2:]), state.clone(), [100], [0], None).double()
    torch.testing.assert_close(kept, want[600:], atol=1e-3, rtol=1e-4)
    lost = ssd_run(sizes, (inputs[0][600:], inputs[1][600:], *inputs[2:]), state * 0, [100], [0], None).double()
    assert float((lost - want[600:]).abs().max()) > 1.0


TALK_SIZES = [  # heads, kv heads, key size, value size, window
    (4, 2, 16, 16, 50), (6, 3, 32, 24, 64), (3, 1, 20, 36, 5), (8, 2, 128, 128, 100), (16, 4, 128, 128, 129), (18, 6, 96, 96, 0),
    (5, 5, 24, 8, 33), (8, 4, 96, 64, 1), (32, 8, 128, 64, 70), (12, 2, 64, 40, 31), (1, 1, 8, 8, 20)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", TALK_SIZES)
def test_attention_with_scores_mixed_over_the_heads(lib, dtype, sizes):
    """Keys and values written by the cache-write kernel into scattered pages, read as a prompt (in query blocks where the
    matrix-core kernel takes the sizes) and as decode steps of one and of several splits.  The last query matches one key
    strongly: placed at the window's last place that key must hold most of a head's weight, a place further none; and the
    first queries share their weight with the sink."""
    from fms_amd.kernels import ops

    H, K, D, V, window = sizes
    gen = torch.Generator().manual_seed(D + V + window)
    n = 200
    base = torch.randn(n, (H + K) * D + K * V, generator=gen)
    talk = torch.eye(H) * 0.5 + torch.randn(H, H, generator=gen) * (0.6 / H ** 0.5)
    talk[0, :] = 0
    talk[0, H - 1] = 1.0  # head 0 looks where the last head's query does
    last, k0 = n - 1, H * D
    per = H // K
    inside = last - window + 1 if window else 0
    scale = 0.3
    visible = P.window(n, window or n)
    table = i32([[5, 0, 3, 6]])
    pos = torch.arange(n, dtype=torch.int32, device=DEV)
    seq = torch.zeros(n, dtype=torch.int32, device=DEV)
    sink = torch.zeros(H, device=DEV)
    tol = dict(atol=5e-5, rtol=1e-4) if dtype == torch.float32 else dict(atol=4e-2, rtol=3e-2)
    for key_at, seen in [(inside, True)] + ([(inside - 1, False)] if window and window < last else []):
        rows = base.clone()
        kv = (H - 1) // per
        key = slice(k0 + kv * D, k0 + (kv + 1) * D)
        rows[key_at, key] *= 4
        q_last = slice((H - 1) * D, H * D)
        rows[last, q_last] = rows[key_at, key] * (60.0 / scale / float(rows[key_at, key] @ rows[key_at, key]))
        rows = rows.to(dtype)
        kc = torch.zeros(8, K, 64, D, dtype=dtype, device=DEV)
        vc = torch.zeros(8, K, V, 64, dtype=dtype, device=DEV)
        qkv = rows.to(DEV).clone()
        ops.rope_kv_write(qkv, pos, seq, table, None, None, 0, kc, vc, H, K, D, V)
        q, k, v = (t.double().view(n, -1, s) for t, s in zip(rows.split([H * D, K * D, K * V], dim=1), (D, D, V)))
        probs = P.softmax_with_null_sink(P.talking_scores(q, k, scale, talk.double()), visible)
        want = torch.stack([probs[h] @ v[:, h // per] for h in range(H)], dim=1)
        assert (float(probs[0][last, key_at]) > 0.9) == seen and (seen or float(probs[0][last, key_at]) == 0.0)
        assert float(probs[:, 0, 0].min()) < 0.95  # the first token shares with the sink
        args = (kc, vc, talk.to(DEV), sink, H, K, D, V, scale, window)
        fits = dtype == torch.bfloat16 and D % 8 == 0 and V % 8 == 0
        qb = {}
        size = ops.talking_qblock(H, K, D, V) if fits else 0
        if size:
            starts = list(range(0, n, size))
            qb = dict(qblock_start=i32(starts), qblock_len=i32([min(size, n - s) for s in starts]), qblock_tokens=size)
        for how in ([qb, dict(force_generic=True)] if fits else [{}]):
            got = ops.talking_attention(qkv, pos, seq, table, *args, **how).double().cpu().view(n, H, V)
            torch.testing.assert_close(got, want, **tol)
        if size and size < n:  # query blocks that start and end anywhere
            starts, at = [], 3
            lens = []
            while at < n:
                starts.append(at)
                lens.append(min(size if len(starts) % 2 else 7, n - at))
                at += lens[-1]
            got = ops.talking_attention(qkv, pos, seq, table, *args, qblock_start=i32(starts), qblock_len=i32(lens),
                                        qblock_tokens=size).double().cpu().view(n, H, V)
            torch.testing.assert_close(got[3:], want[3:], **tol)
        # decode steps over the same cache: the last 40 tokens and the first 3, each a row and a context of its own, and a
        # padding row
        idx = list(range(n - 40, n)) + [0, 1, 2]
        tq = torch.cat([qkv[idx], qkv[:1]])
        tpos = torch.cat([pos[idx], pos[:1]]).contiguous()
        tseq = i32(list(range(len(idx))) + [-1])
        ttable = table.expand(len(idx), -1).contiguous()
        for splits in (0, 1, 2, 5):
            got = ops.talking_attention(tq, tpos, tseq, ttable, *args, decode=True, max_context=n, n_splits=splits).double().cpu().view(-1, H, V)
            torch.testing.assert_close(got[:-1], want[idx], **tol)
            assert float(got[-1].abs().max()) == 0


def test_the_entrance_of_a_pass(lib):
    """x <- W_in [x; x0] + step, from a stream with a scaled branch still to be added."""
    from fms_amd.parts import ConcatLinear, ResidualStream

    class Batch:
        shared = {}

    for width, T in ((48, 5), (36, 3), (64, 300)):
        gen = torch.Generator().manual_seed(width)
        for dtype in (torch.float32, torch.bfloat16):
            part = ConcatLinear(width, 2)
            w, step = torch.randn(width, 2 * width, generator=gen).to(dtype), torch.randn(2, width, generator=gen).to(dtype)
            part.proj.bind("weight", w.to(DEV))
            part.bind("step", step.to(DEV))
            x0 = torch.randn(T, width, generator=gen).to(torch.bfloat16).float()
            stream = ResidualStream(x0.to(DEV).clone())
            part.begin(stream, Batch, dtype)
            branch, scale = torch.randn(T, width, generator=gen).to(dtype), torch.randn(width, generator=gen)
            stream.resid.add_(1.0)  # layers that ran in between
            stream.add_branch(branch.to(DEV), scale=scale.to(DEV))
            x = x0.double() + 1 + branch.double() * scale.double()
            for number in (0, 1):
                part.enter(number, stream, Batch, dtype)
                x = torch.cat([x, x0.double()], dim=1) @ w.double().T + step[number].double()
                assert stream.pending is None and stream.resid.dtype == torch.float32
                tol = dict(atol=1e-3, rtol=1e-4) if dtype == torch.float32 else dict(atol=1.0, rtol=0.05)
                torch.testing.assert_close(stream.resid.double().cpu(), x, **tol)
                x = stream.resid.double().cpu()


# ---- the engine --------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("dtype", DTYPES)
def test_whole_sequence(lib, folders, name, dtype):
    from fms_amd.engine import Engine

    ids, want = expected_for(folders, name, 150, 1, dtype)
    model = get(lib, folders, name, dtype)
    engine = Engine(model, max_tokens=256, max_slots=2)
    slot = engine.new_sequence()
    judge(engine.step([slot], [ids], "all"), want, dtype)
    engine.end_sequence(slot)
    engine.cache.check()


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_the_stream_after_every_layer_run(lib, folders, name):
    """float32: the residual stream after each layer run (a looped layer counts each time) against the plain
    implementation's, so that a fault names its layer."""
    from fms_amd.engine import Engine

    cfg, weights = plain(folders, name)
    ids = tokens_for(cfg["vocab"], 70, 2)
    layers = []
    P.forward(cfg, weights, ids, layers_out=layers)
    model = get(lib, folders, name, "float32")
    seen = []
    blocks = model.layers
    originals = [b.forward for b in blocks]

    def watch(i):
        def forward(stream, batch, cache, act_dtype, next_norm=None):
            originals[i](stream, batch, cache, act_dtype)
            # what is still pending joins the stream in a copy: the stream after this layer
            seen.append(stream.resid.double().cpu() + stream.pending.double().cpu() * stream.pending_scale.double().cpu())
        return forward

    try:
        for i, b in enumerate(blocks):
            b.forward = watch(i)
        engine = Engine(model, max_tokens=128, max_slots=1)
        slot = engine.new_sequence()
        engine.step([slot], [ids], "last")
        engine.end_sequence(slot)
    finally:
        for b in blocks:
            del b.forward
    assert len(seen) == len(layers) == len(P.run_order(cfg))
    for i, got in enumerate(seen):
        torch.testing.assert_close(got, layers[i], atol=5e-4, rtol=1e-4, msg=lambda m, i=i: f"layer run {i}: {m}")


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("dtype", DTYPES)
def test_prompt_then_token_by_token_and_the_first_tokens(lib, folders, name, dtype):
    from fms_amd.engine import Engine

    ids, want = expected_for(folders, name, 150, 1, dtype)
    model = get(lib, folders, name, dtype)
    engine = Engine(model, max_tokens=256, max_slots=2)
    slot = engine.new_sequence()
    got = [engine.step([slot], [ids[:100]], "all")] + [engine.step([slot], [[t]], "last") for t in ids[100:]]
    judge(torch.cat(got), want, dtype)
    engine.end_sequence(slot)
    # from the very first token one by one: empty convolutions and states, the sink against a single key
    slot = engine.new_sequence()
    got = [engine.step([slot], [[t]], "last") for t in ids[:40]]
    judge(torch.cat(got), want[:40], dtype)
    engine.end_sequence(slot)
    engine.cache.check()


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_of_several_sizes(lib, folders, name, dtype):
    from fms_amd.engine import Engine

    ids, want = expected_for(folders, name, 150, 1, dtype)
    model = get(lib, folders, name, dtype)
    engine = Engine(model, max_tokens=256, max_slots=1)
    for cuts in ([2, 2, 60, 1, 63, 2, 20], [64, 64, 22], [63, 2, 2, 83], [1, 127, 22], [2] * 75):
        slot = engine.new_sequence()
        got, at = [], 0
        for n in cuts:
            got.append(engine.step([slot], [ids[at : at + n]], "all"))
            at += n
        assert at == 150
        judge(torch.cat(got), want, dtype)
        engine.end_sequence(slot)
    engine.cache.check()


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("dtype", DTYPES)
def test_ragged_batches_with_pages_and_slots_used_again(lib, folders, name, dtype):
    """Unequal requests in one batch, decoded together; the short ones end early, their slots and pages go to new requests
    that start while the long one goes on (windows give pages back on the way); every request equals itself alone."""
    from fms_amd.engine import Engine

    lens = {"a": (300, 1), "b": (70, 5), "c": (3, 6), "d": (129, 7), "e": (66, 8)}
    reqs = {k: expected_for(folders, name, n, seed, dtype) for k, (n, seed) in lens.items()}
    model = get(lib, folders, name, dtype)
    engine = Engine(model, max_tokens=64 * 9, max_slots=3)
    got = {k: [] for k in reqs}
    slots = {k: engine.new_sequence() for k in ("a", "b", "c")}
    prompt = {"a": 200, "b": 64, "c": 1}
    out = engine.step([slots[k] for k in ("a", "b", "c")], [reqs[k][0][: prompt[k]] for k in ("a", "b", "c")], "all")
    at = 0
    for k in ("a", "b", "c"):
        got[k].append(out[at : at + prompt[k]])
        at += prompt[k]
    done = dict(prompt)
    alive = ["a", "b", "c"]
    waiting = ["d", "e"]
    while alive:
        out = engine.step([slots[k] for k in alive], [[reqs[k][0][done[k]]] for k in alive], "last")
        for i, k in enumerate(alive):
            got[k].append(out[i : i + 1])
            done[k] += 1
        engine.cache.check()
        for k in [k for k in alive if done[k] == len(reqs[k][0])]:
            engine.end_sequence(slots.pop(k))
            alive.remove(k)
        if waiting and len(alive) < 2 and "a" in alive:
            k = waiting.pop(0)
            slots[k] = engine.new_sequence()
            n = len(reqs[k][0]) - 4
            got[k].append(engine.step([slots[k]], [reqs[k][0][:n]], "all"))
            done[k] = n
            alive.append(k)
    assert not waiting
    for k, (ids, want) in reqs.items():
        judge(torch.cat(got[k]), want, dtype)
    engine.cache.check()
    assert engine.cache.n_free_slots == 3 and all(g.pool.n_held == 0 for g in engine.cache.groups)


def with_window(cfg, i, size):
    wrong = json.loads(json.dumps(cfg))
    wrong["layers"][i]["mixer"]["mask"]["size"] = size
    return wrong


@pytest.mark.parametrize("name", ["A", "C"])
def test_the_window_the_sink_and_every_mechanism_decide(lib, name, tmp_path, monkeypatch):
    """Queries scaled up: single keys hold most of a query's weight, among them keys at a window's last place and at page
    borders, in prompts and in decoding.  The plain implementation with a window one token longer or shorter, without the
    sink, with the mixing matrix turned over, and so on, must then differ from the engine by more than the comparison
    allows."""
    from fms_amd.engine import Engine

    folder = write_folder(lib, str(tmp_path / "sharp"), CONFIGS[name], seed=21, sharp=4.0)
    cfg, weights = P.load_model_folder(folder)
    ids = tokens_for(cfg["vocab"], 260, 3)
    want = expect(cfg, weights, ids, "float32")
    model = lib.get_model("hf_pretrained", model_path=folder, data_type="float32")
    for cut in (200, 40):
        engine = Engine(model, max_tokens=384, max_slots=1)
        slot = engine.new_sequence()
        got = [engine.step([slot], [ids[:cut]], "all")] + [engine.step([slot], [[t]], "last") for t in ids[cut:]]
        engine.end_sequence(slot)
        got = torch.cat(got)
        judge(got, want, "float32")

    def must_fail(c, w):
        with pytest.raises(AssertionError):
            judge(got, expect(c, w, ids, "float32"), "float32")

    for i, entry in enumerate(cfg["layers"]):
        if entry["type"] == "attention":
            size = entry["mixer"]["mask"]["size"]
            must_fail(with_window(cfg, i, size + 1), weights)
            must_fail(with_window(cfg, i, size - 1), weights)
            must_fail(cfg, {k: v.T if k == f"l{i}.mix.talk" else v for k, v in weights.items()})
    must_fail(cfg, {k: v.flip(0) if k == "loop.step" else v for k, v in weights.items()})
    must_fail(cfg, {k: v * 0 + 1 if k.endswith((".ls1", ".ls2")) else v for k, v in weights.items()})
    must_fail(dict(cfg, loop=dict(cfg["loop"], times=1)), weights)
    originals = {n: getattr(P, n) for n in ("softmax_with_null_sink", "yarn_frequencies", "gated_group_norm", "over_rms")}
    wrongs = {
        "softmax_with_null_sink": lambda s, visible: torch.softmax(s.masked_fill(~visible, float("-inf")), dim=-1),
        "yarn_frequencies": lambda rot: (originals["yarn_frequencies"](rot)[0], 1.0),
        "gated_group_norm": lambda y, z, w, parts, eps: P.over_rms(y.reshape(y.shape[0], parts, -1), eps).reshape(y.shape) * w * P.silu(z),
        "over_rms": lambda v, eps: v / torch.sqrt((v * v).sum(-1, keepdim=True) + eps),
    }
    for fn, wrong in wrongs.items():
        with monkeypatch.context() as m:
            m.setattr(P, fn, wrong)
            must_fail(cfg, weights)


@pytest.mark.parametrize("name", ["A", "C"])
def test_a_state_lost_after_the_prompt_shows(lib, folders, name):
    """Every pass through a looped layer has a state of its own: each one, set to zero after the prompt, changes the
    logits of the tokens that follow."""
    from fms_amd.engine import Engine

    ids, want = expected_for(folders, name, 150, 1, "float32")
    model = get(lib, folders, name, "float32")
    engine = Engine(model, max_tokens=256, max_slots=1)
    n_states = sum(len(t) for t in engine.cache.state.values())
    assert n_states == 2 * sum(1 for i, _ in P.run_order(plain(folders, name)[0]) if CONFIGS[name]["layers"][i]["type"] != "attention")
    for entry in sorted(engine.cache.state):
        for key in engine.cache.state[entry]:
            slot = engine.new_sequence()
            engine.step([slot], [ids[:140]], "last")
            engine.cache.state[entry][key].zero_()
            got = torch.cat([engine.step([slot], [[t]], "last") for t in ids[140:]])
            engine.end_sequence(slot)
            with pytest.raises(AssertionError):
                judge(got, want[140:], "float32")


def drawn_configuration(seed):
    """A configuration whose every size, count, constant and layer order is drawn at random."""
    import random

    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randint(1, 4)):
        kind = rng.choice(["m", "m", "d", "a"])
        ff = rng.choice([None, 24, 50, 64, 128])
        if kind == "m":
            groups = rng.choice([1, 1, 2, 3])
            heads = groups * rng.choice([1, 2, 3])
            vdim = rng.choice([4, 8, 10, 16, 24, 32, 64])
            norm_groups = rng.choice([g for g in (1, 2, 3, 4, 8) if heads * vdim % g == 0])
            layers.append(layer(mamba(heads, vdim, rng.choice([4, 8, 12, 16, 30, 32, 64, 100, 128]), groups, rng.randint(1, 6), norm_groups), ff))
        elif kind == "d":
            kv = rng.choice([1, 2, 3])
            layers.append(layer(delta(kv * rng.choice([1, 2, 3]), kv, rng.choice([8, 12, 16, 32, 48, 64]), rng.choice([8, 20, 32, 64]),
                                      rng.randint(1, 6)), ff))
        else:
            kv = rng.choice([1, 2, 3, 4])
            dim = rng.choice([8, 16, 20, 32, 48, 64, 80, 96, 128])
            dims = rng.choice([d for d in (2, 4, 8, 12, 16, 24, 32, 48, 64, 128) if d <= dim])
            layers.append(layer(talking(kv * rng.choice([1, 2, 3, 4, 8]), kv, dim, rng.choice([8, 16, 20, 32, 40, 64, 96, 128]), rng.randint(1, 180),
                                        dims, base=rng.choice([100.0, 1e4, 2.5e5]), factor=rng.choice([1.0, 2.0, 8.0, 40.0]),
                                        original=rng.choice([16, 128, 4096]), fast=rng.choice([4.0, 32.0]), slow=rng.choice([0.5, 1.0, 2.0]),
                                        scale=rng.uniform(0.05, 0.3)), ff))
    loop = None
    if rng.random() < 0.8:
        start = rng.randrange(len(layers))
        loop = {"start": start, "stop": rng.randint(start + 1, len(layers)), "times": rng.randint(1, 3)}
    return dict(vocab=rng.randint(50, 600), width=rng.choice([64, 96, 100, 128, 192]), norm={"eps": rng.choice([1e-6, 1e-5, 1e-3])}, loop=loop,
                max_positions=1024, layers=layers)


@pytest.mark.parametrize("seed", range(20))
def test_configurations_drawn_at_random(lib, seed, tmp_path):
    """Every size, constant and layer order drawn: whole, in portions and token by token in float32; whole in bfloat16."""
    from fms_amd.engine import Engine

    folder = write_folder(lib, str(tmp_path / "drawn"), drawn_configuration(seed), seed=100 + seed)
    cfg, weights = P.load_model_folder(folder)
    ids = tokens_for(cfg["vocab"], 180, seed)
    for dtype in DTYPES:
        want = expect(cfg, weights, ids, dtype)
        model = lib.get_model("hf_pretrained", model_path=folder, data_type=dtype)
        engine = Engine(model, max_tokens=256, max_slots=1)
        for cuts in ([180], [70, 1, 2, 107], [130] + [1] * 50):
            slot = engine.new_sequence()
            got, at = [], 0
            for n in cuts:
                got.append(engine.step([slot], [ids[at : at + n]], "all"))
                at += n
            judge(torch.cat(got), want, dtype)
            engine.end_sequence(slot)
        engine.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_through_graphs_and_eager_steps(lib, folders, dtype):
    """200 tokens decoded one by one for three sequences of different lengths, across page borders and past windows, as
    captured graphs and as eager steps: the same logits as the plain implementation's."""
    from fms_amd.engine import Engine
    from fms_amd.sampling import SamplingParams

    name = "C"
    cfg, weights = plain(folders, name)
    model = get(lib, folders, name, dtype)
    seqs = [tokens_for(cfg["vocab"], n, 30 + n) for n in (330, 230, 201)]
    want = [expect(cfg, weights, s, dtype) for s in seqs]
    for use_graphs in (True, False):
        engine = Engine(model, max_tokens=64 * 18, max_slots=3, use_graphs=use_graphs)
        slots = [engine.new_sequence() for _ in seqs]
        engine.step(slots, [s[: len(s) - 200] for s in seqs], "last")
        got = [[] for _ in seqs]
        for i in range(200):
            feed = [s[len(s) - 200 + i] for s in seqs]
            if use_graphs:
                engine.decode_and_choose(slots, feed, SamplingParams(do_sample=False))
                logits = engine.last_graph.logits[: len(seqs)].clone()
            else:
                logits = engine.step(slots, [[t] for t in feed], "last")
            for b in range(len(seqs)):
                got[b].append(logits[b : b + 1])
        for b, s in enumerate(seqs):
            judge(torch.cat(got[b]), want[b][len(s) - 200 :], dtype)
        for s in slots:
            engine.end_sequence(s)
        engine.cache.check()
        assert bool(engine.graph_captures) == use_graphs


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_greedy_generation_through_the_entry_point_and_the_scheduler(lib, folders, name):
    from fms_amd.engine import Engine
    from fms_amd.generation import generate, generate_requests

    cfg, weights = plain(folders, name)
    model = get(lib, folders, name, "float32")
    prompts = [tokens_for(cfg["vocab"], n, 40 + n) for n in (5, 70, 17, 1)]
    want = [P.greedy_generate(cfg, weights, p, 10) for p in prompts]
    for p, w in zip(prompts[:2], want):
        assert generate(model, torch.tensor(p), max_new_tokens=10, do_sample=False).tolist() == p + w
    # the scheduler: more requests than slots, so batches follow one another and slots are used again
    engine = Engine(model, max_tokens=64 * 4, max_slots=2)
    assert generate_requests(engine, prompts, max_new_tokens=10) == want
    stop = want[1][5]
    out = generate_requests(engine, prompts, max_new_tokens=10, stop_token_ids=[stop])
    for o, w in zip(out, want):
        assert o == (w[: w.index(stop) + 1] if stop in w else w)
    engine.cache.check()


def test_command_line_and_trace_replay(lib, folders, tmp_path):
    """The package's programs on a Zimorax folder: the trace replay (float32 and bfloat16, a batch whose requests end
    at different steps) and the registry's view of the architecture."""
    name = "A"
    cfg, weights = plain(folders, name)
    assert "zimorax" in lib.list_models() and "micro" in lib.list_variants("zimorax")
    reqs = {"x": tokens_for(cfg["vocab"], 90, 51), "y": tokens_for(cfg["vocab"], 40, 52)}
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": reqs["x"][:80], "want": [0, 79]}, {"id": "y", "tokens": reqs["y"][:38], "want": [37]}], "end": []}]
    for i in range(10):
        entries = [{"id": "x", "tokens": [reqs["x"][80 + i]], "want": [0]}]
        if i < 2:
            entries.append({"id": "y", "tokens": [reqs["y"][38 + i]], "want": [0] if i == 1 else []})
        steps.append({"step": i + 1, "entries": entries, "end": (["y"] if i == 1 else []) + (["x"] if i == 9 else [])})
    for dtype in DTYPES:
        want = {k: expect(cfg, weights, v, dtype) for k, v in reqs.items()}
        out_dir = str(tmp_path / f"out_{dtype}")
        proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folders[name], "--dtype", dtype,
                               "--out", out_dir, "--max-tokens", "192"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                              capture_output=True, text=True, timeout=110)
        assert proc.returncode == 0, proc.stderr[-2000:]
        assert [line for line in proc.stdout.splitlines() if line.startswith("done ")] == [f"done {i}" for i in range(11)]

        def read(step):
            return torch.from_numpy(np.fromfile(os.path.join(out_dir, f"{step}.f32"), dtype="<f4").reshape(-1, cfg["vocab"]).copy())

        judge(read(0), Expected.stack([want["x"][0], want["x"][79], want["y"][37]]), dtype)
        judge(read(2), Expected.stack([want["x"][81], want["y"][39]]), dtype)
        judge(read(10), want["x"][89:90], dtype)


def test_the_inference_program_and_a_model_from_the_registry(lib, folders):
    """bin/fms_inference with a Zimorax folder (the model class comes from config.json; the text printed is the plain
    implementation's greedy continuation), and a registered variant with random weights through the engine."""
    from fms_amd.engine import Engine
    from fms_amd.tokenizers import CharTokenizer

    name = "A"  # its vocabulary holds the character tokenizer's
    cfg, weights = plain(folders, name)
    tok = CharTokenizer()
    prompt = [ord(c) for c in "once more"]
    new = P.greedy_generate(cfg, weights, prompt, 12)
    if tok.eos_token_id in new:
        new = new[: new.index(tok.eos_token_id)]
    env = dict(os.environ, PYTHONIOENCODING="utf-8")
    cmd = [sys.executable, os.path.join(ROOT, "bin", "fms_inference"), "--architecture", "hf_pretrained", "--model_path", folders[name],
           "--tokenizer", "char_tokenizer", "--default_dtype", "fp32", "--max_new_tokens", "12", "--prompt_ids", ",".join(map(str, prompt))]
    proc = subprocess.run(cmd, stdout=subprocess.PIPE, stderr=subprocess.PIPE, timeout=110, env=env)
    assert proc.returncode == 0, proc.stderr.decode(errors="replace")
    assert tok.decode(prompt + new) in proc.stdout.decode("utf-8")
    model = lib.get_model("zimorax", "micro", data_type="bfloat16", random_seed=5)
    engine = Engine(model, max_tokens=512, max_slots=2)
    slot = engine.new_sequence()
    ids = tokens_for(1024, 300, 9)
    whole = engine.step([slot], [ids], "all")
    engine.end_sequence(slot)
    slot = engine.new_sequence()
    cut = torch.cat([engine.step([slot], [ids[:170]], "all")] + [engine.step([slot], [[t]], "last") for t in ids[170:]])
    engine.end_sequence(slot)
    assert bool(torch.isfinite(whole).all()) and float((whole - cut).abs().max()) < 0.15 * float(whole.abs().max())
