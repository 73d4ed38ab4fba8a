"""Kapuvik on the GPU against the plain implementation (plain_kapuvik.py): every mechanism alone, then the engine
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

import plain_kapuvik as P  # noqa: E402
from gpu_checks import Expected  # noqa: E402

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEV = "cuda"
DTYPES = ["float32", "bfloat16"]
BF16_MARGIN = 3.0
BF16_FURTHER_OFF = 0.02
DRAWS = 4


def parallel(heads, kv, dim, vdim, rheads, rdim, rvdim, rot=None, rrot=None, base=1e4, rbase=2e5, cap=20.0, scale=0.2, scales=(0.8, 1.3), decay=None):
    return {"type": "parallel", "mixer": {
        "left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "rot": {"base": base, "dims": rot or dim}, "scale": scale, "softcap": cap},
        "right": {"heads": rheads, "dim": rdim, "vdim": rvdim, "rot": {"base": rbase, "dims": rrot or rdim},
                  "decay": decay or [1 - 0.5 ** (1 + 9 * h / rheads) for h in range(rheads)]},
        "left_scale": scales[0], "right_scale": scales[1]}}


def latent(heads, dim, rot_dim, vdim, rank, base=5e4, scale=0.15):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "scale": scale,
                                                  "rot": {"base": base, "dims": rot_dim}}}


def gla(heads, dim, vdim, rank, tau=8.0):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "decay_rank": rank}}


def layer(mixer, ff, limit=1.5):
    return dict(mixer, mlp={"kind": "dense", "ff": ff, "limit": limit} if ff else None)


CONFIGS = {
    # values of another size than keys in every mixer, parts of heads rotated, a layer without a feed-forward, a loop of two
    # passes in the middle that holds every kind of mixer
    "A": dict(vocab=300, width=128, embedding={"scale": 2.0}, norm={"eps": 1e-5}, loop={"start": 1, "stop": 4, "times": 2}, logit_softcap=12.0,
              max_positions=1024, layers=[
                  layer(gla(4, 24, 16, 8), 160),
                  layer(parallel(6, 3, 32, 24, 3, 16, 40, rot=16, rrot=8), None),
                  layer(latent(4, 24, 16, 32, 48), 96),
                  layer(gla(2, 16, 40, 12, tau=3.0), 64, limit=0.7),
                  layer(parallel(4, 1, 24, 24, 5, 24, 16), 48),
              ]),
    # sizes that are no multiples of 8 (rows that the matrix instructions cannot load); the loop is the whole model, three
    # passes; one head in places; a rank of one; a decay of one (a plain sum); no cap on the scores
    "B": dict(vocab=257, width=100, embedding={"scale": 1.0}, norm={"eps": 1e-3}, loop={"start": 0, "stop": 3, "times": 3}, logit_softcap=5.0,
              max_positions=1024, layers=[
                  layer(parallel(3, 1, 20, 36, 3, 10, 14, rot=6, rrot=2, base=500.0, cap=None, decay=[0.5, 1.0, 0.97]), 60),
                  layer(gla(3, 10, 7, 1, tau=1.0), 36, limit=5.0),
                  layer(latent(1, 12, 4, 20, 28), None),
              ]),
    # sizes at which bfloat16 runs the matrix-instruction kernels; heads of 128; the loop is one layer, twice
    "C": dict(vocab=512, width=256, embedding={"scale": 0.5}, norm={"eps": 1e-6}, loop={"start": 2, "stop": 3, "times": 2}, logit_softcap=30.0,
              max_positions=2048, layers=[
                  layer(gla(4, 64, 128, 16, tau=16.0), 384, limit=7.0),
                  layer(latent(16, 64, 32, 64, 256, scale=0.1), 256),
                  layer(parallel(8, 2, 128, 128, 4, 128, 64, scale=0.09, cap=50.0), 256),
                  layer(gla(8, 32, 32, 32), None),
              ]),
    # no loop; more than 16 latent heads; key channels above 128; value channels above 256 (no chunks); more than 32 numbers a
    # decay; a cap so low that it bends every score; no cap on the logits
    "D": dict(vocab=400, width=192, embedding={"scale": 3.5}, norm={"eps": 1e-4}, loop=None, logit_softcap=None, max_positions=1024, layers=[
        layer(latent(18, 20, 8, 24, 64), 128),
        layer(gla(2, 200, 72, 70, tau=30.0), 96),
        layer(gla(1, 40, 300, 5), 64),
        layer(parallel(10, 10, 40, 40, 2, 96, 160, rot=4, rrot=96, base=100.0, cap=1.0, scales=(1.0, 1.0)), 64, limit=0.1),
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
    """A model folder with random weights in which every learned number matters: norm weights away from one, biases, slow
    and fast decays, step vectors of some size.  sharp: a factor on the attentions' queries, so that single keys hold most
    of a query's weight.  config.json does not carry the ranks of the decays."""
    from fms_amd.weights import write_safetensors

    lib.write_model_folder(folder, lib.KapuvikConfig(**cfg_kw), seed=seed, architecture="kapuvik", std=0.08)
    path = os.path.join(folder, "config.json")
    with open(path) as f:
        config = json.load(f)
    for entry in config["layers"]:
        entry["mixer"].pop("decay_rank", None)
    with open(path, "w") as f:
        json.dump(config, f)
    cfg, tensors = P.load_model_folder(folder)
    gen = torch.Generator().manual_seed(seed)

    def noise(t, std):
        return torch.randn(t.shape, generator=gen, dtype=torch.float64) * std

    for k in list(tensors):
        t = tensors[k]
        if k.endswith((".norm1", "final.norm")):
            tensors[k] = noise(t, 0.2)
        elif k.endswith((".mix.norm", ".dkv.norm")):
            tensors[k] = 1 + noise(t, 0.2)
        elif k.endswith((".gate.b", ".up.b", ".down.b")):
            tensors[k] = noise(t, 0.3)
        elif k.endswith(".a2.b"):
            tensors[k] = noise(t, 2.0) + 1
        elif k.endswith((".a1", ".a2")):
            tensors[k] = t * 4
        elif k == "loop.step":
            tensors[k] = noise(t, 0.5)
        elif k.endswith(("embed", "head")) or k.endswith((".q", ".k", ".v", ".uk", ".uv", ".gate", ".up")):
            tensors[k] = t * 2
    if sharp != 1.0:
        for i, entry in enumerate(cfg["layers"]):
            for n in {"parallel": ("left.q",), "latent_attention": ("q",)}.get(entry["type"], ()):
                tensors[f"l{i}.mix.{n}"] = tensors[f"l{i}.mix.{n}"] * sharp
    tensors = {k: v.to(torch.bfloat16) for k, v in tensors.items()}
    write_safetensors(os.path.join(folder, "model.safetensors"), [(k, tuple(v.shape), v.dtype) for k, v in tensors.items()],
                      lambda name: tensors[name])
    return folder


@pytest.fixture(scope="module")
def folders(tmp_path_factory, lib):
    return {name: write_folder(lib, str(tmp_path_factory.mktemp(f"kapuvik_{name}")), kw, 3 + i) for i, (name, kw) in enumerate(CONFIGS.items())}


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
    largest over several draws of rounding errors), and its 90th percentile over the sequence; for float32 its own error in
    that type."""
    exact = P.forward(cfg, weights, ids)
    if dtype == "float32":  # a norm over a head's few small entries can be ill-conditioned in that type too
        error = (P.forward(cfg, {k: v.float() for k, v in weights.items()}, ids).double() - exact).abs().amax(dim=-1).float()
        return Expected(exact.float(), error, error)
    exact = exact.float()
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
        error = (got - want.logits).abs()
        allowed = 5e-4 + 1e-3 * want.logits.abs() + 3 * want.ref_error[..., None]
        worst = int(torch.argmax((error / allowed).amax(dim=-1).flatten()))
        assert bool((error <= allowed).all()), (
            f"{int((error > allowed).sum())} of {error.numel()} float32 logits are off, the worst at row {worst}: {float(error.flatten(0, -2)[worst].max()):.4g}; "
            f"the plain implementation in float32 is {float(want.ref_error.flatten()[worst]):.4g} off there")
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
# heads, key channels, value channels, rank of the decays (0: a constant per head), rotated channels
RECURRENCES = [(2, 16, 16, 4, 0), (4, 24, 40, 0, 8), (3, 10, 7, 1, 2), (2, 64, 128, 16, 64), (1, 200, 72, 33, 0), (2, 96, 160, 0, 96), (5, 33, 20, 70, 6),
               (1, 256, 256, 8, 0), (2, 128, 64, 0, 0), (1, 1, 1, 2, 0), (8, 128, 128, 16, 0), (1, 40, 300, 3, 0), (6, 48, 24, 0, 48)]
ROTATION = {"base": 300.0}


class Recurrence:
    """One recurrence's inputs, the plain result and the library's."""

    def __init__(self, sizes, T, seed, bias=(2.0, 1.0), tau=4.0, decay=None, eps=1e-3):
        self.sizes, self.T, self.tau, self.eps = sizes, T, tau, eps
        H, D, V, r, _ = sizes
        gen = torch.Generator().manual_seed(seed)
        self.q, self.k, self.v, self.g = (torch.randn(T, H * n, generator=gen) for n in (D, D, V, V))
        self.low = torch.randn(T, r, generator=gen)
        self.up = torch.randn(H * D, r, generator=gen) / max(r, 1) ** 0.5
        self.bias = torch.randn(H * D, generator=gen) * bias[0] + bias[1]
        self.decay = torch.tensor(decay) if decay is not None else torch.rand(H, generator=gen) * 0.5 + 0.5
        self.norm = 1 + 0.3 * torch.randn(V, generator=gen)

    def part(self, a, b):
        out = object.__new__(Recurrence)
        out.__dict__.update(self.__dict__)
        out.T = b - a
        for n in ("q", "k", "v", "g", "low"):
            setattr(out, n, getattr(self, n)[a:b])
        return out

    def heads(self, positions=None):
        """The plain recurrence's o [T, H, V], before norm and gate."""
        H, D, V, r, rot = self.sizes
        T = self.T
        q, k, v = (x.double().reshape(T, H, -1) for x in (self.q, self.k, self.v))
        if rot:
            pos = torch.arange(T) if positions is None else positions
            q, k = (P.rotate(x, pos, dict(ROTATION, dims=rot), halves=False) for x in (q, k))
        if r:
            z = self.low.double() @ self.up.double().T + self.bias.double()
            decay = (torch.sigmoid(z) ** (1 / self.tau)).reshape(T, H, D)
        else:
            decay = self.decay.double()[None, :, None].expand(T, H, D)
        return P.linear_recurrence(q * D ** -0.5, k, v, decay)

    def want(self, normed=True):
        o = P.over_rms(self.heads(), self.eps) * (self.norm.double() if normed else 1.0)
        return o.reshape(self.T, -1) * P.silu(self.g.double()) * 0.7

    def rows(self):
        """The projection's rows, columns in another order than the library's part has them, some in between unused."""
        pad = torch.full((self.T, 3), float("nan"))
        return torch.cat([self.v, pad, self.low, self.k, self.g, pad, self.q], dim=1)

    def cols(self):
        H, D, V, r, _ = self.sizes
        HD, HV = H * D, H * V
        return (HV + 3 + r + HD + HV + 3, HV + 3 + r, 0, HV + 3 + r + HD, HV + 3)


def run_recurrence(parts, state, slots, starts=None, chunked=None, dtype=torch.float32, normed=True, out=None):
    """The library's recurrence over several sequences at once, from and into `state`."""
    from fms_amd.kernels import ops

    first = parts[0]
    H, D, V, r, rot = first.sizes
    lens = [p.T for p in parts]
    offsets = np.concatenate([[0], np.cumsum(lens)]).tolist()
    starts = starts or [0] * len(parts)
    positions = i32([s + t for s, n in zip(starts, lens) for t in range(n)])
    seq = i32([b for b, n in enumerate(lens) for _ in range(n)])
    kw = {}
    if rot:
        freqs = torch.tensor([ROTATION["base"] ** (-2 * i / rot) for i in range(rot // 2)], dtype=torch.float64).float()
        cos, sin = ops.rope_table(freqs.to(DEV), 4096)
        kw.update(rotation=(cos, sin, rot), positions=positions)
    if r:
        kw.update(up_t=first.up.t().contiguous().to(DEV), up_bias=first.bias.to(DEV), inv_tau=1 / first.tau)
    else:
        kw.update(log_decay=torch.log(first.decay.double()).float().to(DEV))
    return ops.linear_recurrence(torch.cat([p.rows() for p in parts]).to(DEV), first.cols(), H, D, V, state, i32(offsets), seq, i32(slots), len(parts),
                                 max(lens), dtype, q_scale=D ** -0.5, norm_weight=first.norm.to(DEV) if normed else None, eps=first.eps, scale=0.7,
                                 chunked=chunked, out=out, **kw)


@pytest.mark.parametrize("sizes", RECURRENCES)
def test_linear_recurrence_whole_in_portions_and_in_a_batch(lib, sizes):
    """Token by token and in chunks, whole and in portions of any size, a ragged batch in slots that held other sequences:
    all against the plain recurrence."""
    H, D, V, r, rot = sizes
    T = 150
    rec = Recurrence(sizes, T, sum(sizes))
    want = rec.want()
    tol = dict(atol=1e-4, rtol=1e-4)
    long_ok = V <= 256
    for chunked, cuts in ((False, [T]), (long_ok, [T]), (long_ok, [64, 64, 22]), (long_ok, [2, 65, 1, 63, 19]), (False, [1] * 20 + [130]),
                          (None, [100] + [1] * 5 + [2, 2, 41])):
        state = torch.zeros(3, H, V, D, device=DEV)
        got, at = [], 0
        for n in cuts:
            got.append(run_recurrence([rec.part(at, at + n)], state, [1], [at], chunked).cpu())
            at += n
        torch.testing.assert_close(torch.cat(got).double(), want, **tol)
        assert float(state[0].abs().max()) == 0 and float(state[2].abs().max()) == 0
    # a ragged batch into rows of a wider buffer, without a norm weight, in both types
    lens = [70, 1, 64, 15]
    parts = [rec.part(10, 10 + n) for n in lens]
    ends = []
    for chunked in ([True, False] if long_ok else [False]):
        for dtype in (torch.float32, torch.bfloat16):
            state = torch.full((6, H, V, D), 7.0, device=DEV)
            slots = [4, 0, 2, 5]
            state[slots] = 0
            wide = torch.zeros(sum(lens), H * V + 5, dtype=dtype, device=DEV)
            run_recurrence(parts, state, slots, None, chunked, dtype, False, out=wide[:, 3 : 3 + H * V])
            got, at = wide[:, 3 : 3 + H * V].double().cpu(), 0
            for p, n in zip(parts, lens):
                torch.testing.assert_close(got[at : at + n], p.want(normed=False), **(tol if dtype == torch.float32 else dict(atol=2e-3, rtol=1e-2)))
                at += n
            assert float((state[[1, 3]] - 7).abs().max()) == 0 and float(wide[:, :3].abs().max()) == 0 == float(wide[:, 3 + H * V :].abs().max())
            ends.append(state.cpu())
    for other in ends[1:]:
        torch.testing.assert_close(other, ends[0], atol=2e-4, rtol=1e-4)


def test_padding_rows_of_a_decode_step_become_zeros_and_touch_no_state(lib):
    from fms_amd.kernels import ops

    sizes = (3, 16, 24, 4, 0)
    rec = Recurrence(sizes, 4, 1)
    state = torch.randn(2, 3, 24, 16, device=DEV)
    before = state.clone()
    kw = dict(up_t=rec.up.t().contiguous().to(DEV), up_bias=rec.bias.to(DEV), inv_tau=0.25)
    out = ops.linear_recurrence(rec.rows().to(DEV), rec.cols(), 3, 16, 24, state, i32([0, 1, 2, 3, 4]), i32([0, -1, 2, -1]), i32([1, 0, 0, 1]), 4, 1,
                                torch.bfloat16, out=torch.full((4, 72), 9.0, dtype=torch.bfloat16, device=DEV), **kw)
    assert float(out[[1, 3]].abs().max()) == 0 and float(out[[0, 2]].abs().min(dim=1).values.max()) > 0
    assert bool(torch.isfinite(state).all()) and not torch.equal(state, before)
    only = before.clone()
    ops.linear_recurrence(rec.rows()[[0, 2]].to(DEV), rec.cols(), 3, 16, 24, only, i32([0, 1, 2]), i32([0, 1]), i32([1, 0]), 2, 1, torch.bfloat16, **kw)
    assert torch.equal(only, state)


@pytest.mark.parametrize("rank", [0, 4])
def test_linear_recurrence_far_tokens_and_a_lost_state(lib, rank):
    """A decay of 0.9999 a token carries the first token across 700; a state lost between two steps shows."""
    sizes = (2, 16, 24, rank, 0)
    T = 700
    rec = Recurrence(sizes, T, 5, decay=[0.9999, 0.9995])
    rec.up, rec.bias = rec.up * 0, torch.full_like(rec.bias, float(np.log(0.9996 / 0.0004)))
    far = rec.part(0, T)
    far.v = far.v * 1e-3
    far.v[0] *= 1e6
    far.q = far.q * 0 + 1
    far.k = far.k * 0.1
    far.k[0] = 1
    without = far.part(0, T)
    without.v = without.v.clone()
    without.v[0] = 0
    want = far.want()
    assert float((far.heads() - without.heads())[-1].abs().max()) > 50 * float(without.heads()[-1].abs().max())  # the first token is what shows
    for chunked in (True, False):
        got = run_recurrence([far], torch.zeros(1, 2, 24, 16, device=DEV), [0], chunked=chunked).cpu().double()
        torch.testing.assert_close(got, want, atol=1e-4, rtol=1e-4)
    state = torch.zeros(1, 2, 24, 16, device=DEV)
    want = rec.want()
    run_recurrence([rec.part(0, 600)], state, [0])
    kept = run_recurrence([rec.part(600, T)], state.clone(), [0]).cpu().double()
    torch.testing.assert_close(kept, want[600:], atol=3e-4, rtol=1e-3)
    lost = run_recurrence([rec.part(600, T)], state * 0, [0]).cpu().double()
    assert float((lost - want[600:]).abs().max()) > 0.3


def test_decays_that_vanish_next_to_decays_of_nearly_one(lib):
    """Channels whose decay is exp(-40) or exactly zero at some tokens beside channels that keep everything: quotients of
    running products would leave the range, neighbours must stay exact, and the state must forget what the decay forgets."""
    sizes = (2, 72, 40, 3, 0)
    T = 200
    for strength, tau in ((40.0, 1.0), (300.0, 1.0), (30.0, 16.0), (3000.0, 16.0)):
        rec = Recurrence(sizes, T, int(strength), tau=tau, bias=(3.0, 6.0))
        z = torch.where((torch.arange(T) % 7 == 3)[:, None], torch.tensor(-strength), torch.tensor(2.0))
        rec.low = z * torch.tensor([1.0, 0.0, 0.0])
        rec.up = torch.zeros_like(rec.up)
        rec.up[::3, 0] = 1.0  # every third channel follows it
        rec.eps = 1e-6
        want = rec.want()
        assert bool(torch.isfinite(want).all())
        for chunked in (True, False, None):
            got = run_recurrence([rec], torch.zeros(1, 2, 40, 72, device=DEV), [0], chunked=chunked).cpu().double()
            torch.testing.assert_close(got, want, atol=2e-4, rtol=1e-3)
        # the decays' exactness beside one another, token by token: what the state holds
        states = []
        for chunked in (True, False):
            state = torch.zeros(1, 2, 40, 72, device=DEV)
            run_recurrence([rec], state, [0], chunked=chunked)
            states.append(state.cpu())
        torch.testing.assert_close(states[0], states[1], atol=2e-5, rtol=1e-4)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows", [1, 7, 16, 17, 40, 130, 192, 193, 300])
def test_the_clamped_gated_product(lib, dtype, rows):
    """min(gate, limit) and clamp(up) with biases, at sizes of every kernel that forms it, into rows of a wider buffer; with
    values on both sides of both limits."""
    from fms_amd.kernels import ops

    gen = torch.Generator().manual_seed(rows)
    for width, hidden, limit in ((64, 48, 1.5), (96, 200, 0.4), (50, 33, 3.0), (512, 1056, 2.0)):
        x = torch.randn(rows, width, generator=gen).to(dtype)
        w, b = (torch.randn(2 * hidden, width, generator=gen) * 3 / width ** 0.5).to(dtype), (torch.randn(2 * hidden, generator=gen) * 0.5).to(dtype)
        pre = x.double() @ w.double().T
        m = {"limit": limit}
        ident = {"gate": torch.eye(hidden, dtype=torch.float64), "up": torch.eye(hidden, dtype=torch.float64), "down": torch.eye(hidden, dtype=torch.float64)}
        g, u = pre[:, :hidden] + b[:hidden].double(), pre[:, hidden:] + b[hidden:].double()
        assert float(g.max()) > limit and float(u.max()) > limit and float(u.min()) < -limit and float(g.min()) < -limit
        zero = torch.zeros(hidden, dtype=torch.float64)
        clamp = ops.GateClamp(limit, 1.702, 1.0)
        want = torch.stack([P.feed_forward(torch.cat([gi, ui]), {"gate": torch.cat([ident["gate"], 0 * ident["gate"]], 1), "gate.b": zero,
                                                                "up": torch.cat([0 * ident["up"], ident["up"]], 1), "up.b": zero,
                                                                "down": ident["down"], "down.b": zero}, m) for gi, ui in zip(g[:5], u[:5])])
        wide = torch.zeros(rows, hidden + 13, dtype=dtype, device=DEV)
        got = ops.gated_linear(x.to(DEV), w.to(DEV), b.to(DEV), "silu", clamp=clamp, out=wide[:, 8 : 8 + hidden])
        tol = dict(atol=2e-4, rtol=1e-4) if dtype == torch.float32 else dict(atol=6e-2, rtol=3e-2)
        torch.testing.assert_close(got[:5].double().cpu(), want, **tol)
        every = torch.clamp(g, max=limit) * torch.sigmoid(1.702 * torch.clamp(g, max=limit)) * (torch.clamp(u, -limit, limit) + 1)
        torch.testing.assert_close(got.double().cpu(), every, **tol)
        assert float(wide[:, :8].abs().max()) == 0 == float(wide[:, 8 + hidden :].abs().max())
        # the ordinary gated unit into such rows
        got = ops.gated_linear(x.to(DEV), w.to(DEV), b.to(DEV), "silu", out=wide[:, 8 : 8 + hidden])
        torch.testing.assert_close(got.double().cpu(), P.silu(g) * u, **(tol if dtype == torch.float32 else dict(atol=0.15, rtol=3e-2)))


def test_capped_logits_and_the_entrance_of_a_pass(lib):
    """cap * tanh(logit / cap) over values far beyond the cap; x + x0 + step (x0 not in the first pass), from a stream with a
    branch still to be added, and x0 as it was whatever layers add to the stream in between."""
    from fms_amd.kernels import ops
    from fms_amd.parts import AddEmbedding, ResidualStream

    x = torch.linspace(-300, 300, 7003)
    torch.testing.assert_close(ops.soft_cap_(x.to(DEV).clone(), 15.0).cpu().double(), P.soft_cap(x.double(), 15.0), atol=2e-5, rtol=1e-5)

    class Batch:
        shared = {}

    for width, T, at_start in ((48, 5, False), (37, 3, True), (64, 300, False), (2048, 9, True)):
        gen = torch.Generator().manual_seed(width)
        for dtype in (torch.float32, torch.bfloat16):
            part = AddEmbedding(width, 3, at_start=at_start)
            step = torch.randn(3, width, generator=gen).to(dtype)
            part.bind("step", step.to(DEV))
            part.finalize(DEV, dtype)
            x0 = torch.randn(T, width, generator=gen)
            stream = ResidualStream(x0.to(DEV).clone())
            part.begin(stream, Batch, dtype)
            want = x0.double()
            if not at_start:
                stream.resid.add_(1.0)  # layers that run before the first pass
                want = want + 1
            for number in range(3):
                branch = torch.randn(T, width, generator=gen).to(dtype)
                if number or not at_start:
                    stream.add_branch(branch.to(DEV))
                    want = want + branch.double()
                part.enter(number, stream, Batch, dtype)
                want = want + (x0.double() if number else 0.0) + step[number].double()
                assert stream.pending is None and stream.resid.dtype == torch.float32
                torch.testing.assert_close(stream.resid.double().cpu(), want, atol=1e-5, rtol=1e-5)
                stream.resid.add_(0.5)  # a layer of the pass adds in place
                want = want + 0.5


def test_norms_that_store_their_scale_around_zero(lib):
    from fms_amd.parts import make_part

    gen = torch.Generator().manual_seed(3)
    for width in (50, 320, 2048):
        norm = make_part("norm", "rmsnorm", width=width, eps=1e-3, weight_offset=1.0)
        w = torch.randn(width, generator=gen) * 0.2
        norm.bind("weight", w.to(DEV))
        norm.finalize(DEV, torch.float32)
        x = torch.randn(4, width, generator=gen) * 0.05  # eps counts
        got = norm.add_norm(x.to(DEV).clone(), None, torch.float32)
        torch.testing.assert_close(got.cpu().double(), P.zero_centred_norm(x.double(), w.double(), 1e-3), atol=1e-5, rtol=1e-5)


ATTENTIONS = [(4, 2, 16, 16, 0.0), (6, 3, 48, 48, 8.0), (3, 1, 20, 36, 2.0), (8, 2, 128, 128, 30.0), (5, 5, 24, 8, 1.0), (16, 1, 64, 64, 5.0), (8, 4, 96, 64, 3.0)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", ATTENTIONS)
def test_capped_attention_far_keys_and_page_borders(lib, dtype, sizes):
    """Keys and values of other sizes, capped scores, scattered pages; the last query matches one key strongly, far away and
    on both sides of page borders, as a prompt and as decode steps."""
    from fms_amd.kernels import ops

    H, K, D, V, cap = sizes
    gen = torch.Generator().manual_seed(D + V)
    n, scale = 200, 0.3
    base = torch.randn(n, (H + K) * D + K * V, generator=gen)
    last, k0, per = n - 1, H * D, H // K
    pos = torch.arange(n, dtype=torch.int32, device=DEV)
    seq = torch.zeros(n, dtype=torch.int32, device=DEV)
    table = i32([[5, 0, 3, 6]])
    tol = dict(atol=2e-4, rtol=1e-4) if dtype == torch.float32 else dict(atol=0.1, rtol=4e-2)
    for key_at in (0, 63, 64, 127, 128, 198, 199):
        rows = base.clone()
        key = slice(k0, k0 + D)
        rows[key_at, key] *= 4
        rows[key_at, k0 + K * D : k0 + K * D + V] *= 20  # and its value tells
        score = min(60.0, 3.0 * cap if cap else 60.0)
        rows[last, :D] = rows[key_at, key] * (score / scale / float(rows[key_at, key] @ rows[key_at, key]))
        rows = rows.to(dtype)
        kc = torch.zeros(8, K, 64, D, dtype=dtype, device=DEV)
        vc = torch.zeros(8, K, V, 64, dtype=dtype, device=DEV)
        qkv = rows.to(DEV).clone()
        ops.rope_kv_write(qkv, pos, seq, table, None, None, 0, kc, vc, H, K, D, V)
        q, k, v = (t.double().view(n, -1, s) for t, s in zip(rows.split([H * D, K * D, K * V], dim=1), (D, D, V)))
        probs = [P.softmax_over(P.soft_cap((q[:, h] @ k[:, h // per].T) * scale, cap), P.causal(n)) for h in range(H)]
        want = torch.stack([probs[h] @ v[:, h // per] for h in range(H)], dim=1)
        others = probs[0][last].clone()
        others[key_at] = 0
        assert float(probs[0][last, key_at]) > (1.2 if cap and cap < 20 else 10) * float(others.max())
        args = (kc, vc, H, K, D, scale, 0)
        size = ops.prefill_qblock(H, K, D, n) if dtype == torch.bfloat16 and D % 16 == 0 and V == D and not ops.prefill_cap_is_generic(D, cap) else 0
        kw = {}
        if size:
            starts = list(range(0, n, size))
            kw = dict(qblock_start=i32(starts), qblock_len=i32([min(size, n - s) for s in starts]), qblock_tokens=size)
        got = ops.attention(qkv, pos, seq, table, *args, decode=False, max_context=n, soft_cap=cap, value_dim=V, **kw)
        torch.testing.assert_close(got.double().cpu().view(n, H, V), want, **tol)
        idx = list(range(n - 20, n)) + [0, 1]
        got = ops.attention(qkv[idx].contiguous(), pos[idx].contiguous(), i32(list(range(len(idx)))), table.expand(len(idx), -1).contiguous(), *args,
                            decode=True, max_context=n, soft_cap=cap, value_dim=V, row_order=i32(list(range(len(idx)))))
        torch.testing.assert_close(got.double().cpu().view(-1, H, V), want[idx], **tol)


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
            seen.append(stream.resid.double().cpu() + stream.pending.double().cpu())  # what is still pending joins in a copy
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
    # from the very first token one by one: empty states, a single key
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
    for cuts in ([2, 2, 60, 1, 63, 2, 20], [64, 64, 22], [63, 2, 2, 83], [1, 127, 22], [31, 32, 33, 54], [2] * 75):
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
    that start while the long one goes on; every request equals itself alone."""
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
            # the newcomer's prompt in a step in which the long request goes on by a token
            out = engine.step([slots["a"], slots[k]], [[reqs["a"][0][done["a"]]], reqs[k][0][:n]], "all")
            got["a"].append(out[:1])
            done["a"] += 1
            got[k].append(out[1:])
            done[k] = n
            alive.append(k)
    assert not waiting
    for k, (ids, want) in reqs.items():
        judge(torch.cat(got[k]), want, dtype)
    engine.cache.check()
    assert engine.cache.n_free_slots == 3 and all(g.pool.n_held == 0 for g in engine.cache.groups)


def changed(cfg, *path_and_value):
    """A copy of the configuration with one entry replaced, found by its path."""
    *path, value = path_and_value
    out = json.loads(json.dumps(cfg))
    at = out
    for key in path[:-1]:
        at = at[key]
    at[path[-1]] = value
    return out


@pytest.mark.parametrize("name", ["A", "C"])
def test_every_mechanism_and_far_keys_decide(lib, name, tmp_path, monkeypatch):
    """Queries scaled up: single keys hold most of a query's weight, among them far ones and ones at page borders, in prompts
    and in decoding.  The plain implementation with one mechanism changed must then differ from the engine by more than the
    comparison allows."""
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

    def must_fail(c, w, tokens=ids, rows=slice(None)):
        with pytest.raises(AssertionError):
            judge(got[rows], expect(c, w, tokens, "float32")[rows], "float32")

    # the first tokens are still seen by the last ones: other tokens there change logits more than 200 tokens on
    must_fail(cfg, weights, [(t + 1) % cfg["vocab"] for t in ids[:3]] + ids[3:], slice(210, None))
    for i, entry in enumerate(cfg["layers"]):
        m, p = entry["mixer"], f"l{i}.mix."
        at = ("layers", i, "mixer")
        if entry["type"] == "parallel":
            must_fail(changed(cfg, *at, "left", "softcap", m["left"]["softcap"] * 2), weights)
            must_fail(changed(cfg, *at, "left", "rot", "base", m["left"]["rot"]["base"] * 2), weights)
            must_fail(changed(cfg, *at, "right", "rot", "base", m["right"]["rot"]["base"] * 4), weights)
            must_fail(changed(cfg, *at, "right", "decay", m["right"]["decay"][::-1]), weights)
            must_fail(changed(cfg, *at, "left_scale", m["right_scale"]), weights)
            must_fail(changed(cfg, *at, "right_scale", m["left_scale"]), weights)
        elif entry["type"] == "latent_attention":
            must_fail(changed(cfg, *at, "rot", "base", m["rot"]["base"] * 4), weights)
            must_fail(cfg, {k: v * 0 + 1 if k == p + "dkv.norm" else v for k, v in weights.items()})
        else:
            must_fail(changed(cfg, *at, "tau", m["tau"] * 1.1), weights)
            must_fail(cfg, {k: v * 0 if k == p + "a2.b" else v for k, v in weights.items()})
            must_fail(cfg, {k: v * 0 + 1 if k == p + "norm" else v for k, v in weights.items()})
        if entry["mlp"]:
            must_fail(changed(cfg, "layers", i, "mlp", "limit", entry["mlp"]["limit"] * 0.8), weights)
            must_fail(cfg, {k: v * 0 if k == f"l{i}.mlp.down.b" else v for k, v in weights.items()})
    must_fail(changed(cfg, "embedding", "scale", cfg["embedding"]["scale"] * 1.05), weights)
    must_fail(changed(cfg, "logit_softcap", cfg["logit_softcap"] * 1.1), weights)
    must_fail(changed(cfg, "loop", "times", 1), weights)
    must_fail(cfg, {k: v.flip(0) if k == "loop.step" else v for k, v in weights.items()})
    must_fail(cfg, {k: v * 0 if k == "final.norm" else v for k, v in weights.items()})
    originals = {n: getattr(P, n) for n in ("rotate", "over_rms", "feed_forward", "silu")}
    wrongs = {
        "rotate": lambda v, pos, rot, halves: originals["rotate"](v, pos, rot, not halves),
        "over_rms": lambda v, eps: v / torch.sqrt((v * v).sum(-1, keepdim=True) + eps),
        "feed_forward": lambda h, w, m: originals["feed_forward"](h, dict(w, **{"up.b": w["up.b"] - 1}), dict(m, limit=m["limit"])),
        "silu": torch.sigmoid,
    }
    for fn, wrong in wrongs.items():
        with monkeypatch.context() as patch:
            patch.setattr(P, fn, wrong)
            must_fail(cfg, weights)


@pytest.mark.parametrize("name", ["A", "C"])
def test_a_state_lost_after_the_prompt_shows(lib, folders, name):
    """Every pass through a looped layer has a state of its own: each one, set to zero after the prompt, changes the
    logits of the tokens that follow."""
    from fms_amd.engine import Engine

    ids, want = expected_for(folders, name, 150, 1, "float32")
    model = get(lib, folders, name, "float32")
    engine = Engine(model, max_tokens=256, max_slots=1)
    assert len(engine.cache.state) == sum(1 for i, _ in P.run_order(plain(folders, name)[0]) if CONFIGS[name]["layers"][i]["type"] != "latent_attention")
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
    even = [2, 4, 8, 12, 16, 24, 32, 48, 64, 128]
    for _ in range(rng.randint(1, 4)):
        kind = rng.choice(["p", "p", "l", "g", "g"])
        ff = rng.choice([None, 24, 50, 64, 128])
        limit = rng.choice([0.3, 1.0, 7.0])
        if kind == "p":
            kv = rng.choice([1, 2, 3, 4])
            dim = rng.choice([8, 16, 20, 32, 48, 64, 80, 96, 128])
            vdim = rng.choice([dim, dim, 8, 20, 32, 64, 128])
            rdim = rng.choice([2, 8, 10, 16, 32, 48, 64, 100])
            mixer = parallel(kv * rng.choice([1, 2, 3, 4, 8]), kv, dim, vdim, rng.choice([1, 2, 3, 5]), rdim, rng.choice([4, 8, 20, 32, 64, 128]),
                             rot=rng.choice([d for d in even if d <= dim]), rrot=rng.choice([d for d in even if d <= rdim]),
                             base=rng.choice([100.0, 1e4, 2.5e5]), rbase=rng.choice([50.0, 1e6]), cap=rng.choice([2.0, 10.0, 50.0]),
                             scale=rng.uniform(0.05, 0.3), scales=(rng.uniform(0.5, 1.5), rng.choice([1.0, 0.7])))
        elif kind == "l":
            rot = rng.choice([2, 4, 8, 16, 32, 64])
            mixer = latent(rng.choice([1, 2, 4, 5, 16, 20]), rng.choice([8, 12, 20, 32, 64]), rot, rng.choice([8, 12, 20, 32, 64]),
                           rng.choice([16, 28, 32, 64, 96, 128, 256]), base=rng.choice([100.0, 1e4, 2.5e5]), scale=rng.uniform(0.05, 0.3))
        else:
            mixer = gla(rng.choice([1, 2, 3, 4]), rng.choice([4, 8, 12, 16, 33, 64, 100, 128]), rng.choice([4, 8, 20, 32, 64, 128]),
                        rng.choice([1, 3, 8, 16, 40]), tau=rng.choice([1.0, 4.0, 16.0, 50.0]))
        layers.append(layer(mixer, ff, limit))
    loop = None
    if rng.random() < 0.8:
        start = rng.randrange(len(layers))
        loop = {"start": start, "stop": rng.randint(start + 1, len(layers)), "times": rng.randint(1, 3)}
    return dict(vocab=rng.randint(50, 600), width=rng.choice([64, 96, 100, 128, 192]), embedding={"scale": rng.choice([1.0, 0.3, 4.0])},
                norm={"eps": rng.choice([1e-6, 1e-5, 1e-3])}, loop=loop, logit_softcap=rng.choice([4.0, 20.0, None]), max_positions=1024, layers=layers)


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
    """200 tokens decoded one by one for three sequences of different lengths, across page borders, as captured graphs and
    as eager steps: the same logits as the plain implementation's."""
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
    """The package's programs on a Kapuvik folder: the trace replay (float32 and bfloat16, a batch whose requests end
    at different steps) and the registry's view of the architecture."""
    name = "A"
    cfg, weights = plain(folders, name)
    assert "kapuvik" in lib.list_models() and "micro" in lib.list_variants("kapuvik")
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
    """bin/fms_inference with a Kapuvik folder (the model class comes from config.json; the text printed is the plain
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
    model = lib.get_model("kapuvik", "micro", data_type="bfloat16", random_seed=5)
    engine = Engine(model, max_tokens=512, max_slots=2)
    slot = engine.new_sequence()
    ids = tokens_for(1024, 300, 9)
    whole = engine.step([slot], [ids], "all")
    engine.end_sequence(slot)
    slot = engine.new_sequence()
    cut = torch.cat([engine.step([slot], [ids[:170]], "all")] + [engine.step([slot], [[t]], "last") for t in ids[170:]])
    engine.end_sequence(slot)
    assert bool(torch.isfinite(whole).all()) and float((whole - cut).abs().max()) < 0.15 * float(whole.abs().max())
