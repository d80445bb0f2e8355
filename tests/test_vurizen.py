"""Vurizen through the engine (model registry, latent cache with shared rows and matrix states,
state slots, Engine.step, generation) against the plain float64 statement in ``oracle_vurizen.py``,
on small random checkpoints of several shapes. Every case runs on the CPU (PyTorch statements of
the ops) and, marked ``gpu``, on the HIP kernels in fp32 and bf16.
"""
import json
import math
import os

import pytest
import torch
from safetensors.torch import save_file

import oracle_vurizen as O
from theroundtaible_amd.engine import Engine, EngineConfig, SamplingParams, Turn
from theroundtaible_amd.engine.kv_cache import KVCacheOOM, LatentKVCache
from theroundtaible_amd.models.config import GLASpec, LatentAttentionSpec, MoESpec, config_from_dir, get_config, parse_vurizen
from theroundtaible_amd.models.weights import layout_for
from theroundtaible_amd.ops import hybrid as Hy
from theroundtaible_amd.ops import latent as L

GPU = pytest.mark.gpu
RUNS = [("cpu", "fp32"), pytest.param(("cuda:0", "fp32"), marks=GPU), pytest.param(("cuda:0", "bf16"), marks=GPU)]
YARN = {"factor": 6.0, "original": 64, "fast": 16.0, "slow": 1.0}


def moe(experts=6, top=2, ff=24, count=3, keep=2, scale=1.7):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}, "scale": scale}}


def lat(heads=3, dim=10, rot_dim=8, vdim=6, kv_rank=20, window=11, kv_from=None, base=10000.0, scaling=YARN, scale=None,
        mlp="moe"):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "mask": {"size": window},
         "rot": {"base": base, "dims": rot_dim}, "scale": 1.3 * (dim + rot_dim) ** -0.5 if scale is None else scale}
    if scaling is not None:
        m["rot"]["scaling"] = scaling
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": moe() if mlp == "moe" else mlp}


def gla(heads=2, dim=6, vdim=10, tau=8.0, mlp="moe"):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau},
            "mlp": moe(4, 3, 16, 2, 2, 0.8) if mlp == "moe" else mlp}


def make_config(width=40, vocab=97, layers=None, mult=0.6, eps=1e-5):
    if layers is None:
        layers = [lat(), gla(), lat(5, 7, 8, 12, 20, window=6, kv_from=0, mlp=moe(5, 1, 20, 1, 1, 1.2)), gla(3, 9, 4, 2.0, None),
                  lat(2, 12, 4, 8, 16, window=17, scaling=None, mlp=None), lat(4, 5, 4, 3, 16, window=30, kv_from=4, scaling=None)]
    return {"architecture": "Vurizen", "layers": layers, "norm": {"eps": eps}, "residual_mult": mult, "vocab": vocab,
            "width": width}


def config_like(cfg):
    return parse_vurizen(cfg, "t")


def settle(cfg, run):
    """bf16 runs choose every expert: rounding would otherwise flip a close router call now and
    then. The routing weights still count; the choice itself is covered by the fp32 runs and the
    router's own test."""
    if run[1] != "bf16":
        return cfg
    cfg = json.loads(json.dumps(cfg))
    for layer in cfg["layers"]:
        if layer["mlp"] is not None:
            r = layer["mlp"]["router"]
            r["top"] = r["experts"]
            r["groups"]["keep"] = r["groups"]["count"]
    return cfg


def make_checkpoint(path, cfg, seed=0, edit=None):
    """Random weights for ``cfg`` (a config.json dict) written as a checkpoint directory; returns
    the float64 tensors. ``edit(P)`` may change tensors before they are written."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    mc = config_from_dir(path)
    g = torch.Generator().manual_seed(seed)
    P = {}
    for name, (shape, _, _) in layout_for(mc).items():
        shape = tuple(5 if n < 0 else n for n in shape)        # the decay path's rank is the checkpoint's
        if name.endswith(("norm1.b", "norm2.b", "final.norm.b")):
            w = 0.5 * torch.randn(shape, generator=g)
        elif name.endswith("norm"):
            w = 0.6 + torch.rand(shape, generator=g)
        elif name.endswith(("norm1", "norm2")):
            w = 0.6 + torch.rand(shape, generator=g)
        elif name.endswith(("ls1", "ls2")):
            w = (0.4 + torch.rand(shape, generator=g)) * torch.sign(torch.randn(shape, generator=g))
        elif name.endswith("a2.b"):                 # decays from quick to almost none
            w = 1.5 * torch.randn(shape, generator=g)
        elif name.endswith("correction"):           # choice scores of both signs
            w = torch.randn(shape, generator=g) - 0.6
        elif name == "embed":
            w = torch.randn(shape, generator=g)
        elif name.endswith("router"):               # clear choices: no top-k call is close
            w = torch.randn(shape, generator=g) * 2.5 / math.sqrt(shape[-1])
        else:
            w = torch.randn(shape, generator=g) / math.sqrt(shape[-1])
        P[name] = w.to(torch.bfloat16).float()      # values both number formats hold exactly
    if edit is not None:
        edit(P)
    save_file({k: v.contiguous() for k, v in P.items()}, os.path.join(path, "model.safetensors"))
    return {k: v.double() for k, v in P.items()}


def engine_for(path, run, tokens=512, block_size=16, slots=4, graphs=False):
    device, dtype = run
    if device != "cpu":     # the GPU cases fail loudly when an extension is missing
        Hy.native()
        L.native()
    return Engine(EngineConfig(model=str(path), weights=str(path), dtype=dtype, device=device, block_size=block_size,
                               num_blocks=(tokens + block_size - 1) // block_size + (1 if graphs else 0),
                               use_graphs=graphs, state_slots=slots, max_batch=slots))


def close(got, want, run, what=""):
    """fp32 runs: every logit within 1e-3 of the oracle. bf16 runs: every row within 6 % of the
    logits' range and half of the rows within 2 % (a wrong kernel misses by about the whole range)."""
    got = got.double().cpu()
    if run[1] != "bf16":
        torch.testing.assert_close(got, want, msg=lambda m: f"{what}: {m}", rtol=0, atol=1e-3)
        return
    err, span = (got - want).abs().max(-1).values, float(want.abs().max())
    assert torch.isfinite(got).all(), what
    assert float(err.median()) < 0.02 * span and float(err.max()) < 0.06 * span, \
        f"{what}: median row error {float(err.median()):.3f}, worst {float(err.max()):.3f}, range {span:.1f}"


def toks(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def dev_of(run):
    return torch.device(run[0])


def dt_of(run):
    return torch.bfloat16 if run[1] == "bf16" else torch.float32


def spans(cuts, slot=1):
    """Row metadata of ONE sequence fed in portions: yields (rows, positions, start_pos, cu_q, slots)."""
    at = 0
    for n in cuts:
        yield (slice(at, at + n), torch.arange(at, at + n), torch.tensor([at], dtype=torch.int32),
               torch.tensor([0, n], dtype=torch.int32), torch.tensor([slot], dtype=torch.int32))
        at += n


# ---- each mechanism alone (package ops against the oracle's functions) ----------------------------

@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("W", [24, 333, 2048, 5000])
def test_layer_norm_with_the_scaled_add(run, W):
    """x += y * s, then the layer norm of the sum; rows with a mean far from zero (a variance taken
    as E[x^2] - mean^2 would lose its digits there), and rows wider than a workgroup keeps."""
    dev, dt = dev_of(run), dt_of(run)
    g = torch.Generator().manual_seed(W)
    x = torch.randn(5, W, generator=g) + torch.tensor([0.0, 3.0, -200.0, 900.0, 0.1])[:, None]
    y, s = torch.randn(5, W, generator=g).to(dt).float(), torch.randn(W, generator=g)
    w, b = 0.6 + torch.rand(W, generator=g), torch.randn(W, generator=g)
    xs = x.double() + y.double() * s.double()
    xd = x.clone().to(dev)
    got = Hy.add_layer_norm(xd, y.to(dt).to(dev), s.to(dev), w.to(dev), b.to(dev), 1e-3, dt)
    assert float((xd.double().cpu() - xs).abs().max()) < 2e-4
    want = O.layer_norm(xs, w.double(), b.double(), 1e-3)
    assert float((got.double().cpu() - want).abs().max()) < (0.05 if run[1] == "bf16" else 2e-3)
    xd = x.clone().to(dev)
    got = Hy.add_layer_norm(xd, None, s.to(dev), w.to(dev), b.to(dev), 1e-3, dt)        # nothing pending
    assert torch.equal(xd.cpu(), x)
    want = O.layer_norm(x.double(), w.double(), b.double(), 1e-3)
    assert float((got.double().cpu() - want).abs().max()) < (0.05 if run[1] == "bf16" else 2e-3)


def test_rotary_tables():
    """Plain and blended frequencies, ramps of several entries, of a single step, and an upper end
    below the lower one."""
    for rot in ({"base": 5000.0, "dims": 16}, {"base": 300.0, "dims": 24, "scaling": YARN},
                {"base": 300.0, "dims": 8, "scaling": {"factor": 2.0, "original": 16, "fast": 2.0, "slow": 2.0}},
                {"base": 20.0, "dims": 4, "scaling": {"factor": 3.0, "original": 4096, "fast": 1.0, "slow": 64.0}},
                {"base": 1e6, "dims": 2, "scaling": {"factor": 8.0, "original": 100, "fast": 32.0, "slow": 1.0}}):
        spec = config_like(make_config(layers=[lat(rot_dim=rot["dims"], base=rot["base"], scaling=rot.get("scaling"))]))
        t = L.rotary_table(spec.layers[0].mixer.rot, "cpu")
        want, mag = O.rotary_frequencies(rot)
        assert float(((t.freq.double() - want).abs() / want).max()) < 1e-6 and abs(t.mag - mag) < 1e-12 and t.halves
    assert L.rotary_table(None, "cpu").freq is None


def _latent_case(run, m, n, seed, edit=None):
    """Projected columns [3 spare | q | latent + key part], key / value up-projections, norm weight."""
    g = torch.Generator().manual_seed(seed)
    nq, C, R = m["heads"] * (m["dim"] + m["rot_dim"]), m["kv_rank"], m["rot_dim"]
    proj = torch.randn(n, nq + C + R, generator=g)
    uk = torch.randn(m["heads"] * m["dim"], C, generator=g) / math.sqrt(C)
    uv = torch.randn(m["heads"] * m["vdim"], C, generator=g) / math.sqrt(C)
    w = 0.6 + torch.rand(C, generator=g)
    if edit is not None:
        edit(proj, nq, uk)
    return tuple(t.to(dt_of(run)).float() for t in (proj, uk, uv, w))


def _run_latent(run, m, case, cuts, BS, splits=3):
    """latent_prep + latent_attention of one sequence through a paged cache whose pages are
    scattered; decoded rows on split keys."""
    proj, uk, uv, w = case
    dev, dt = dev_of(run), dt_of(run)
    spec = config_like(make_config(layers=[{"type": "latent_attention", "mixer": m, "mlp": None}])).layers[0].mixer
    H, D, R, V, C = spec.heads, spec.dim, spec.rot_dim, spec.vdim, spec.kv_rank
    nq, n = H * (D + R), proj.shape[0]
    table = L.rotary_table(spec.rot, dev)
    nb = (n + BS - 1) // BS
    perm = torch.randperm(nb + 3, generator=torch.Generator().manual_seed(5))[:nb].to(torch.int32)
    rows = torch.zeros(nb + 3, BS, C + R, dtype=dt, device=dev)
    bt = perm[None].to(dev)
    uk_h, uv_ht = uk.view(H, D, C).to(dt).to(dev), uv.view(H, V, C).transpose(1, 2).contiguous().to(dt).to(dev)
    out = torch.zeros(n, H, V)
    for r, pos, sp, cu, sl in spans(cuts):
        T = r.stop - r.start
        slot_map = (perm[pos // BS].long() * BS + pos % BS).to(dev)
        p = proj[r].to(dt).to(dev)
        L.latent_prep(p, spec, None, w.to(dev), 1e-5, pos.to(dev), rows, slot_map, dt, kv_off=nq, table=table)
        q = p[:, :nq].unflatten(1, (H, D + R))
        q_lat = torch.bmm(q[:, :, :D].transpose(0, 1), uk_h)
        one = T == 1 and r.start > 0 and dev.type == "cuda"
        o = L.latent_attention(q_lat, q, spec, rows, bt, cu.to(dev), sp.to(dev), None, num_splits=splits if one else 1,
                               out_dtype=dt, table=table)
        out[r] = torch.bmm(o, uv_ht).transpose(0, 1).float().cpu()
    return out.reshape(n, H * V).double()


def _oracle_latent(m, case):
    """The oracle's attention with identity projections: h = the projected columns themselves."""
    proj, uk, uv, w = (t.double() for t in case)
    nq, N = m["heads"] * (m["dim"] + m["rot_dim"]), proj.shape[1]
    eye = torch.eye(N, dtype=torch.float64)
    P = {"q": eye[:nq], "dkv": eye[nq:], "dkv.norm": w, "uk": uk, "uv": uv,
         "o": torch.eye(m["heads"] * m["vdim"], dtype=torch.float64)}
    return O.latent_attention(proj, P, "", m, O.latent_rows(proj, P, "", m, 1e-5))


LATENT_SIZES = [dict(heads=3, dim=10, rot_dim=8, vdim=6, kv_rank=20), dict(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=3),
                dict(heads=6, dim=24, rot_dim=16, vdim=20, kv_rank=64), dict(heads=40, dim=8, rot_dim=32, vdim=8, kv_rank=192),
                dict(heads=2, dim=40, rot_dim=6, vdim=72, kv_rank=300), dict(heads=70, dim=8, rot_dim=16, vdim=4, kv_rank=128)]


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("size", range(len(LATENT_SIZES)))
@pytest.mark.parametrize("cuts", [[150], [5, 1, 1, 2, 60, 1, 7, 2, 71]])
def test_latent_attention(run, size, cuts):
    """Several head counts and widths (matrix-core shapes among them), a window that crosses key
    tiles, prompts, portions down to two tokens and decoded rows."""
    m = lat(**LATENT_SIZES[size], window=70)["mixer"]
    case = _latent_case(run, m, sum(cuts), size)
    got, want = _run_latent(run, m, case, cuts, 8), _oracle_latent(m, case)
    assert float((got - want).abs().max()) < (0.06 if run[1] == "bf16" else 2e-4)


@pytest.mark.parametrize("run", RUNS)
def test_partly_rotated_key_part(run):
    """A rotation over fewer entries than the rotated part: the rest pass as they are."""
    m = lat(2, 8, 12, 6, 16, window=9)["mixer"]
    m["rot"]["dims"] = 6
    case = _latent_case(run, m, 40, 3)
    got, want = _run_latent(run, m, case, [22, 1, 1, 16], 8), _oracle_latent(m, case)
    assert float((got - want).abs().max()) < (0.06 if run[1] == "bf16" else 2e-4)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("kv_rank,rot_dim", [(20, 4), (64, 16)])
@pytest.mark.parametrize("window", [1, 2, 16, 17, 64, 65, 130])
def test_window_edges_with_a_key_that_stands_out(run, kv_rank, rot_dim, window):
    """A few keys dominate every query that still sees them, so a window that is one token too wide
    or too narrow changes a row by far more than the tolerance: rows just inside and just outside
    every edge, in a prompt, in portions cut at the edge, and decoded; both attention kernels."""
    n, BS = 240, 16
    m = lat(2, 8, rot_dim, 6, kv_rank, window=window, scale=1.0)["mixer"]
    loud = {3: 40.0, 40: 8.0, 63: 6.0, 64: 5.0, 100: 4.0}       # an earlier one drowns the later ones

    def edit(proj, nq, uk):
        # the unrotated key is entry 0 of the latent: small for every token, large for the loud ones
        D = 8 + rot_dim
        uk.zero_()
        uk[0, 0] = uk[8, 0] = 1.0
        proj[:, [0, D]] = 12.0                       # unrotated query entry that meets it, both heads
        proj[:, nq] = 0.0
        for a in range(2):
            proj[:, a * D + 8:a * D + 8 + rot_dim] *= 0.1
        for j, v in loud.items():
            proj[j, nq] = v
    case = _latent_case(run, m, n, 2, edit)
    want = _oracle_latent(m, case)
    if window > 1:
        for j in (3, 100):              # the edge shows in the oracle itself
            assert float((want[j + window - 1] - want[j + window]).abs().max()) > 0.3
    e = 100 + window - 1
    for cuts in ([n], [min(e, 238), 1, 1] + ([n - e - 2] if n - e - 2 > 0 else []), [4, 62] + [2] * 30 + [1] * 114):
        got = _run_latent(run, m, case, cuts, BS)
        assert float((got - want).abs().max()) < (0.06 if run[1] == "bf16" else 3e-4), cuts


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("kv_rank", [24, 128])
def test_a_far_key_among_hundreds(run, kv_rank):
    """A window of 900 over 700 tokens on scattered pages: one early key carries almost all the
    weight of the last rows, as a prompt, in portions, and decoded on 2 to 32 key ranges."""
    n = 700
    m = lat(3, 8, 16, 12, kv_rank, window=900, scale=1.0)["mixer"]

    def edit(proj, nq, uk):
        uk.zero_()
        uk[[0, 8, 16], 0] = 1.0
        proj[:, [0, 24, 48]] = 10.0
        proj[:, nq] = 0.0
        proj[17, nq] = 25.0
        for a in range(3):
            proj[:, a * 24 + 8:a * 24 + 24] *= 0.1
    case = _latent_case(run, m, n, 4, edit)
    want = _oracle_latent(m, case)
    for cuts, splits in (([n], 1), ([699, 1], 2), ([64, 300, 2, 333, 1], 32), ([690] + [1] * 10, 7)):
        got = _run_latent(run, m, case, cuts, 16, splits)
        assert float((got - want)[-12:].abs().max()) < (0.06 if run[1] == "bf16" else 3e-4), (cuts, splits)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("tau", [1.0, 16.0])
@pytest.mark.parametrize("n,rank", [(3, 1), (9, 5), (300, 16)])
def test_gla_preparation(run, tau, n, rank):
    """Scaled queries, keys, values, and the decays of the low-rank path: biases far to both sides
    give decays at 0 and at 1 without overflow."""
    dev, dt = dev_of(run), dt_of(run)
    A, D, V = 3, 7, 5
    g = torch.Generator().manual_seed(n)
    proj = torch.randn(n, 2 + 2 * A * D + A * V + rank + 4, generator=g).to(dt).float()
    a2, ab = torch.randn(A * D, rank, generator=g), 2 * torch.randn(A * D, generator=g)
    ab[0], ab[1] = -150.0, 150.0
    k0, v0, a0 = 2 + A * D, 2 + 2 * A * D, 2 + 2 * A * D + A * V
    got = Hy.gla_prep(proj.to(dt).to(dev), GLASpec(A, D, V, tau), 2, k0, v0, a0, a2.t().contiguous().to(dev), ab.to(dev))
    eye = torch.eye(rank, dtype=torch.float64)
    want = O.gla_decay(proj[:, a0:a0 + rank].double(), {"a1": eye, "a2": a2.double(), "a2.b": ab.double()}, "",
                       {"heads": A, "dim": D, "tau": tau}).reshape(n, A * D)
    assert float((got[0].double().cpu() - proj[:, 2:k0].double() * D ** -0.5).abs().max()) < 1e-6
    assert torch.equal(got[1].cpu(), proj[:, k0:v0]) and torch.equal(got[3].cpu(), proj[:, v0:a0])
    assert torch.isfinite(got[2]).all() and float((got[2].double().cpu() - want).abs().max()) < 2e-6


@pytest.mark.parametrize("run", RUNS[:2])
@pytest.mark.parametrize("A,D,V", [(2, 6, 10), (1, 64, 64), (3, 72, 20), (1, 130, 33)])
@pytest.mark.parametrize("cuts", [[33], [200], [64, 65, 1, 1, 2, 128], [1, 2, 130, 1, 63]])
def test_gla_recurrence(run, A, D, V, cuts):
    """The scan with a decay per key channel — decays of exactly 0 and 1 among them — in one go, in
    portions, decoded, and (spans longer than a chunk, on the GPU) in parallel chunks; the slot it
    starts in holds another sequence's state."""
    dev = dev_of(run)
    n = sum(cuts)
    g = torch.Generator().manual_seed(n + D)
    q, k = torch.randn(n, A * D, generator=g) * D ** -0.5, torch.randn(n, A * D, generator=g)
    v, w = torch.randn(n, A * V, generator=g), torch.rand(n, A * D, generator=g) ** 0.1
    w[::7, 1] = 0.0
    w[:, 2] = 1.0
    want = O.gla_scan(*(t.double().reshape(n, A, -1) for t in (q, k, v, w))).reshape(n, A * V)
    for chunked in (False, True) if dev.type == "cuda" else (False,):
        state = torch.full((3, A * D * V), 5.0, device=dev)
        got = []
        for r, pos, sp, cu, sl in spans(cuts):
            ch = Hy.scan_chunks(cu, dev) if chunked else None
            got.append(Hy.state_scan(*(t[r].to(dev) for t in (q, k, v, w)), None, None, None, state, cu.to(dev), sp.to(dev),
                                     sl.to(dev), A, D, V, chunks=ch))
        err = (torch.cat(got).double().cpu() - want).abs().max()
        assert float(err) < 2e-4 * max(1.0, float(want.abs().max())), f"chunked={chunked}"
        assert float((state[[0, 2]] - 5.0).abs().max()) == 0


@GPU
def test_chunked_scan_of_unequal_sequences():
    """Long and short spans, new and continued sequences, in one launch of chunks; constant decays too."""
    A, D, V, lens = 2, 32, 48, [150, 1, 64, 65, 200]
    g = torch.Generator().manual_seed(3)
    n = sum(lens)
    cu = torch.tensor([0] + torch.tensor(lens).cumsum(0).tolist(), dtype=torch.int32)
    sp = torch.tensor([0, 7, 64, 0, 3], dtype=torch.int32)
    slots = torch.tensor([2, 0, 5, 3, 1], dtype=torch.int32)
    q, k, w = torch.randn(n, A * D, generator=g), torch.randn(n, A * D, generator=g), torch.rand(n, A * D, generator=g) ** 0.2
    v, st = torch.randn(n, A * V, generator=g), torch.randn(6, A * D * V, generator=g)
    dec = torch.tensor([0.9, 0.5])
    for ww, dd in ((w, None), (None, dec)):
        s0 = st.clone()
        want = Hy.ref_state_scan(q, k, v, ww, None, None, dd, s0, cu, sp, slots, A, D, V)
        s1 = st.clone().cuda()
        ch = Hy.scan_chunks(cu, "cuda:0")
        got = Hy.state_scan(q.cuda(), k.cuda(), v.cuda(), ww.cuda() if ww is not None else None, None, None,
                            dd.cuda() if dd is not None else None, s1, cu.cuda(), sp.cuda(), slots.cuda(), A, D, V, chunks=ch)
        torch.testing.assert_close(got.cpu(), want, rtol=2e-4, atol=2e-4)
        torch.testing.assert_close(s1.cpu(), s0, rtol=2e-4, atol=2e-4)


ROUTERS = [(6, 2, 3, 2, 1.7), (8, 3, 4, 3, 0.5), (5, 2, 1, 1, 1.0), (4, 1, 4, 2, 1.0), (9, 3, 3, 1, 2.5), (1, 1, 1, 1, 1.0),
           (96, 8, 8, 3, 1.0), (130, 6, 65, 40, 1.3)]


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("E,top,count,keep,scale", ROUTERS)
def test_router(run, E, top, count, keep, scale):
    """Choices by score + correction within the best groups, weights by the score alone; choice
    scores of both signs (a masked expert must lose to any negative score too), groups of one expert, one
    group, more experts than a wave has lanes."""
    dev, dt = dev_of(run), dt_of(run)
    g = torch.Generator().manual_seed(E)
    n, W = 50, 36
    h = torch.randn(n, W, generator=g).to(dt).float()
    wr, corr = torch.randn(E, W, generator=g) * 0.4, torch.randn(E, generator=g) * 0.5 - 1.2
    spec = MoESpec(E, top, 8, score="sigmoid", groups=count, group_keep=keep, scale=scale)
    idx, wt = Hy.route_groups(h.to(dt).to(dev), wr.to(dev), spec, corr.to(dev))
    r = {"experts": E, "top": top, "groups": {"count": count, "keep": keep}, "scale": scale}
    pick, weights = O.route(h.double(), wr.double(), corr.double(), r)
    assert idx.shape == (n, top)
    plain = O.route(h.double(), wr.double(), torch.zeros(E, dtype=torch.float64), r)[0]
    if E > 4:       # the correction decides some of the choices
        assert plain != pick
    for t in range(n):
        order = sorted(range(top), key=lambda j: pick[t][j])
        mine = sorted(range(top), key=lambda j: int(idx[t, j]))
        assert [pick[t][j] for j in order] == [int(idx[t, j]) for j in mine]
        for a, b in zip(order, mine):
            assert abs(weights[t][a] - float(wt[t, b])) < 1e-4


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("n", [1, 5, 40])
def test_experts(run, n):
    dev, dt = dev_of(run), dt_of(run)
    g = torch.Generator().manual_seed(n)
    E, top, W, Fw = 6, 2, 40, 24
    mlp = moe(E, top, Fw, 3, 2, 1.3)
    P = {"router": torch.randn(E, W, generator=g), "correction": torch.randn(E, generator=g)}
    for e in range(E):
        for nm, sh in (("gate", (Fw, W)), ("up", (Fw, W)), ("down", (W, Fw))):
            P[f"e{e}.{nm}"] = torch.randn(sh, generator=g).to(dt).float() / math.sqrt(sh[1])
    P = {k: v.to(dt).float() for k, v in P.items()}
    h = torch.randn(n, W, generator=g).to(dt).float()
    want = O.moe_ff(h.double(), {k: v.double() for k, v in P.items()}, "", mlp)
    spec = config_like(make_config(layers=[gla(mlp=mlp)])).layers[0].moe
    hd = h.to(dt).to(dev)
    idx, wt = Hy.route_groups(hd, P["router"].to(dev), spec, P["correction"].to(dev))
    w_gu = torch.stack([torch.cat([P[f"e{e}.gate"], P[f"e{e}.up"]]) for e in range(E)]).to(dt).to(dev)
    w_down = torch.stack([P[f"e{e}.down"] for e in range(E)]).to(dt).to(dev)
    for by_row in (True, False):
        tol = 0.06 if run[1] == "bf16" else 1e-4
        got = Hy.moe_experts(hd, idx, wt, w_gu, w_down, dt, by_row=by_row)
        assert float((got.double().cpu() - want).abs().max()) < tol, by_row
        # the same rows left to the launch that adds and norms them, for all rows and for some
        res = Hy.moe_experts(hd, idx, wt, w_gu, w_down, dt, by_row=by_row, combine=False)
        s, one = torch.linspace(-1, 1, W), torch.ones(W, device=dev)
        for rows in (torch.arange(n), torch.tensor([n - 1, 0])):
            x = torch.zeros(len(rows), W, device=dev)
            Hy.add_layer_norm(x, res.select(rows.to(dev)) if len(rows) != n else res, s.to(dev), one, one, 1e-5, dt)
            assert float((x.double().cpu() - want[rows] * s.double()).abs().max()) < tol, by_row


@GPU
@pytest.mark.parametrize("T,E,top,W,F", [(300, 4, 2, 128, 96), (129, 8, 3, 72, 200), (17, 5, 5, 40, 24), (700, 3, 1, 264, 136),
                                         (33, 70, 4, 64, 64), (260, 1, 1, 64, 72)])
def test_grouped_experts_on_the_matrix_cores(T, E, top, W, F):
    """The grouped products at sizes off the tile shapes — experts without rows, experts with more
    than one tile, widths that end inside a tile or a K step — against plain products."""
    g = torch.Generator().manual_seed(T)
    h = torch.randn(T, W, generator=g).bfloat16()
    w_gu = (torch.randn(E, 2 * F, W, generator=g) / W ** 0.5).bfloat16()
    w_down = (torch.randn(E, W, F, generator=g) / F ** 0.5).bfloat16()
    idx = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)]).to(torch.int32)
    if E > 2:
        idx[idx == 1] = 1 if top > E - 1 else 0          # (one expert of several keeps no row; a row may name one twice)
    wt = torch.rand(T, top, generator=g)
    want = torch.zeros(T, W, dtype=torch.float64)
    for e in range(E):
        a = h.double() @ w_gu[e].double().T
        y = (torch.nn.functional.silu(a[:, :F]) * a[:, F:]) @ w_down[e].double().T
        want += y * (wt.double() * (idx == e)).sum(1, keepdim=True)
    args = [t.cuda() for t in (h, idx, wt, w_gu, w_down)]
    a = Hy.moe_experts(*args, torch.float32, by_row=False)
    b = Hy.moe_experts(*args, torch.float32, by_row=False)
    assert float((a.double().cpu() - want).abs().max()) < 0.05
    assert torch.equal(a, b)                            # rows do not depend on their place
    alone = Hy.moe_experts(args[0][5:6], args[1][5:6], args[2][5:6], args[3], args[4], torch.float32, by_row=False)
    assert torch.equal(alone[0], a[5])


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("T,H,K,N", [(1, 3, 8, 5), (8, 4, 64, 192), (17, 2, 40, 16), (32, 5, 200, 70)])
def test_head_product(run, T, H, K, N):
    """Per-head products of a few rows, from a column range of a wider projection into head-major
    rows and back."""
    dev, dt = dev_of(run), dt_of(run)
    g = torch.Generator().manual_seed(K)
    proj = torch.randn(T, H * (K + 8) + 16, generator=g).to(dt).to(dev)
    w = (torch.randn(H, N, K, generator=g) / K ** 0.5).to(dt).to(dev)
    x = proj[:, :H * (K + 8)].unflatten(1, (H, K + 8))[:, :, :K]
    want = torch.einsum("thk,hnk->thn", x.double().cpu(), w.double().cpu())
    if run == ("cuda:0", "fp32"):
        assert not L.head_product_fits(x, w)        # fp32 layers use library products
        return
    a = torch.full((H, T, N), 9.0, dtype=dt, device=dev)
    L.head_product(x, w, a.transpose(0, 1))
    b = torch.full((T, H, N), 9.0, dtype=dt, device=dev)
    L.head_product(x, w, b)
    tol = 0.03 if run[1] == "bf16" else 1e-4
    assert float((a.double().cpu().transpose(0, 1) - want).abs().max()) < tol
    assert float((b.double().cpu() - want).abs().max()) < tol


# ---- the model through the engine -----------------------------------------------------------------

def test_registry_and_config():
    """Sizes, constants and branches come from config.json; what it does not have is off; impossible
    combinations are refused."""
    cfg = config_like(make_config())
    a, b = cfg.layers[0].mixer, cfg.layers[2].mixer
    assert isinstance(a, LatentAttentionSpec) and (a.window, a.kv_from, a.q_rank, a.rot.halves) == (11, None, 0, True)
    assert (b.kv_from, b.heads, b.window) == (0, 5, 6) and cfg.layers[1].mixer == GLASpec(2, 6, 10, 8.0)
    assert cfg.layers[0].moe == MoESpec(6, 2, 24, score="sigmoid", groups=3, group_keep=2, scale=1.7)
    assert cfg.layers[3].ff == 0 and cfg.residual_mult == 0.6 and cfg.kv_bytes_per_token(2) == 2 * (28 + 20)
    bare = lat(scaling=None)
    del bare["mixer"]["mask"], bare["mixer"]["rot"]
    bare["mlp"] = {"expert": {"ff": 8}, "router": {"experts": 3, "top": 1}}
    got = config_like(make_config(layers=[bare])).layers[0]
    assert (got.mixer.window, got.mixer.rot, got.moe.groups, got.moe.scale) == (0, None, 1, 1.0)
    for bad in ([lat(kv_from=0)], [gla(), lat(kv_from=0)], [lat(), lat(kv_from=0), lat(kv_from=1)],
                [lat(), lat(kv_rank=24, kv_from=0)], [lat(), lat(base=77.0, kv_from=0)], [lat(window=0)],
                [lat(mlp=moe(6, 2, 8, 4, 2))], [lat(mlp=moe(6, 5, 8, 3, 2))], [dict(lat(), type="other")]):
        with pytest.raises(ValueError):
            config_like(make_config(layers=bad))
    assert get_config("tiny-vurizen").arch == "vurizen"


def test_shared_rows_in_the_cache():
    """A layer that reads another's rows has the same tensor; block copies touch it once; a fork
    copies the matrix states."""
    c = LatentKVCache([6, None, 6, None], 8, 0, 5, 4, "cpu", torch.float32, n_slots=3, shared=[None, None, 0, None],
                      rec_widths=[0, 7, 0, 9])
    assert c.rows[2] is c.rows[0] and c.rows[1] is None and len(c.state_tensors()) == 2
    c.rows[0][1] = 3.0
    c.copy_blocks([1], [4])
    assert float(c.rows[2][4].min()) == 3.0
    s = c.seq("a")
    c.ensure_capacity(s, 5)
    s.tokens.extend(range(5))
    c.rec[1][c.slot_of(s)] = 2.5
    s.state_len = 5
    f = c.fork("a", "b", copy=True)
    assert f.slot != s.slot and float(c.rec[1][f.slot].min()) == 2.5
    assert LatentKVCache.bytes_per_block([6, None, None], 4, 2) == 48


@pytest.mark.parametrize("run", RUNS)
def test_whole_prompt_and_layers(tmp_path, run):
    cfg = settle(make_config(), run)
    P = make_checkpoint(tmp_path / "m", cfg, seed=1)
    e = engine_for(tmp_path / "m", run)
    t = toks(45, cfg["vocab"], 1)
    layers = []
    want = O.forward(cfg, P, t, layers)
    got = e.step([("a", t, list(range(len(t))))])
    close(got, want, run, "logits")
    s = e.kv.seq("b")
    tok, pos, meta = e._varlen_meta([e.reserve(s, t)])
    keep = []
    with torch.no_grad():
        e.model.forward(tok, pos, e.kv, meta, keep_layers=keep)
    assert len(keep) == len(layers) == 6
    for i, (a, b) in enumerate(zip(keep, layers)):
        err = float((a.double().cpu() - b).abs().max())
        assert err < (0.06 * float(b.abs().max()) if run[1] == "bf16" else 1e-3), f"residual stream after layer {i}: {err}"


SHAPES = {
    # one head, one expert, windows of one token, constants that are 1
    "ones": [lat(1, 1, 2, 1, 1, window=1, scaling=None, scale=1.0, mlp=moe(1, 1, 3, 1, 1, 1.0)), gla(1, 1, 1, 1.0, None),
             lat(1, 2, 2, 1, 1, window=1, kv_from=0, scaling=None, mlp=None)],
    # only recurrent layers: no pages at all
    "gla-only": [gla(4, 5, 3), gla(1, 12, 20, 3.0, None)],
    # several layers over the same rows, none in between; every expert chosen
    "shared": [lat(2, 6, 4, 9, 24, window=5), lat(3, 8, 4, 4, 24, window=40, kv_from=0), lat(1, 3, 4, 16, 24, window=2, kv_from=0,
               mlp=moe(4, 4, 9, 2, 2)), lat(6, 4, 4, 5, 24, window=64, kv_from=0, mlp=None)],
    # heads wider than a wave's 64 lanes, states of 72 x 132 and 130 x 70, a latent wider than 256
    "wide": [lat(2, 72, 20, 70, 264, window=33, mlp=None), gla(1, 72, 132, 16.0, None), gla(2, 130, 70, 4.0, None)],
    # more heads than one attention workgroup's pairs
    "many-heads": [lat(70, 3, 4, 2, 12, window=20), gla(9, 4, 4)],
    # more experts than a wave's lanes, groups of one expert
    "experts": [gla(2, 4, 4, mlp=moe(66, 5, 7, 11, 3)), lat(mlp=moe(5, 2, 11, 5, 3, 0.3))],
}


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("shape", list(SHAPES))
def test_other_sizes(tmp_path, run, shape):
    """Sizes and constants that the usual test model makes equal or 1."""
    one = shape == "ones"
    cfg = settle(make_config(width=24, vocab=61, layers=SHAPES[shape], mult=1.0 if one else 0.35, eps=1e-3), run)
    P = make_checkpoint(tmp_path / "m", cfg, seed=2)
    e = engine_for(tmp_path / "m", run, block_size=8)
    t = toks(90, cfg["vocab"], 2)
    want = O.forward(cfg, P, t)
    got = torch.cat([e.step([("a", t[:57], list(range(57)))]), e.step([("a", t[57:59], [0, 1])])] +
                    [e.step([("a", t[i:i + 1], [0])]) for i in range(59, 90)])
    if one and run[1] == "bf16":        # a norm over a single entry is a sign: rounding flips some
        assert float((got.double().cpu() - want).abs().max(-1).values.median()) < 0.02 * float(want.abs().max())
    else:
        close(got, want, run, shape)


@pytest.mark.parametrize("run", RUNS)
def test_wider_layers(tmp_path, run):
    """Rows wide enough for several waves per workgroup, sizes of the matrix-core attention kernel,
    64-wide recurrence heads, a window that crosses many key tiles and pages: a prompt in portions
    (some span many scan chunks), then decoded tokens."""
    layers = [lat(8, 32, 32, 64, 192, window=200, mlp=moe(8, 2, 128, 4, 2)), gla(4, 64, 64, 16.0, moe(8, 2, 128, 4, 2)),
              lat(16, 32, 32, 32, 192, window=90, kv_from=0, mlp=moe(8, 2, 128, 4, 2))]
    cfg = settle(make_config(width=512, vocab=331, layers=layers), run)
    P = make_checkpoint(tmp_path / "m", cfg, seed=21)
    e = engine_for(tmp_path / "m", run, tokens=1024, block_size=32)
    t = toks(520, cfg["vocab"], 21)
    want = O.forward(cfg, P, t)
    got = [e.step([("a", t[:300], [0, 199, 200, 201, 299])]), e.step([("a", t[300:302], [0, 1])]),
           e.step([("a", t[302:500], [0, 197])])] + [e.step([("a", t[i:i + 1], [0])]) for i in range(500, 520)]
    rows = [0, 199, 200, 201, 299, 300, 301, 302, 499] + list(range(500, 520))
    close(torch.cat(got), want[rows], run, "wider layers")


@pytest.mark.parametrize("run", RUNS)
def test_window_edges_and_far_keys_through_the_engine(tmp_path, run):
    """One token id whose key stands out, at positions whose windows end at page and tile borders:
    the rows just inside and just outside every edge, in prompts, in portions and decoded. The layer
    that shares the rows has the wider window, so the key it still sees has left the first layer's."""
    window, wide, loud = 48, 130, 7
    layers = [lat(1, 8, 16, 8, 64, window=window, scale=1.0, mlp=None),
              lat(1, 8, 16, 8, 64, window=wide, kv_from=0, scale=1.0, mlp=None)]
    cfg = make_config(width=32, vocab=64, layers=layers, mult=0.9)

    def edit(P):
        P["embed"][:, 0] = -1.0          # channel 0 of the norm's output tells the loud token from the others
        P["embed"][loud] *= 0.1
        P["embed"][loud, 0] = 8.0
        for i in (0, 1):
            p = f"l{i}.mix."
            P[p + "q"].mul_(0.05)
            P[p + "uk"].zero_()
            P[p + "uk"][0, 0] = 1.0
            P[f"l{i}.norm1.b"][5] = 4.0
            P[p + "q"][0, 5] = 4.0       # a query entry that is large for every token
        P["l0.mix.dkv"][0] = 0.0
        P["l0.mix.dkv"][0, 0] = 3.0
        P["l0.ls1"][0] = 0.0
    P = make_checkpoint(tmp_path / "m", cfg, seed=31, edit=edit)
    n = 300
    t = [x if x != loud else 8 for x in toks(n, 64, 31)]
    for j in (16, 63, 128):
        t[j] = loud
    want = O.forward(cfg, P, t)
    edges = sorted({j + w + d for j in (16, 63, 128) for w in (window, wide) for d in (-2, -1, 0, 1) if j + w + d < n})
    t2 = list(t)
    t2[128] = 9                         # without the loud key, rows that saw it change
    other = O.forward(cfg, P, t2)
    assert float((other - want)[128 + window - 1].abs().max()) > 0.3
    assert float((other - want)[128 + wide - 1].abs().max()) > 0.3
    assert float((other - want)[128 + wide:].abs().max()) < 1e-9      # the shared rows come from the first layer
    e = engine_for(tmp_path / "m", run, tokens=1024, block_size=16)
    whole = e.step([("w", t, edges)], end=["w"])
    close(whole, want[edges], run, "prompt")
    for name, cuts in (("cut at edges", [16 + window, 2, 63 + window - 66, 1, 1, 65, 120]), ("decoded", [60] + [1] * 240),
                       ("pairs", [2] * 150)):
        got, at = [], 0
        for c in cuts:
            c = min(c, n - at)
            if c > 0:
                got.append(e.step([("a", t[at:at + c], list(range(c)))]))
                at += c
        e.release("a")
        close(torch.cat(got)[edges], want[edges], run, name)


# ---- portions, decoding, batches ------------------------------------------------------------------

@pytest.mark.parametrize("run", RUNS)
def test_prefill_against_token_by_token(tmp_path, run):
    cfg = settle(make_config(), run)
    P = make_checkpoint(tmp_path / "m", cfg, seed=3)
    e = engine_for(tmp_path / "m", run)
    t = toks(40, cfg["vocab"], 3)
    want = O.forward(cfg, P, t)
    one = torch.cat([e.step([("a", [x], [0])]) for x in t])          # from the first token on
    close(one, want, run, "token by token")
    whole = e.step([("b", t, list(range(40)))])
    close(whole, want, run, "whole")
    if run[1] != "bf16":
        assert float((one - whole).abs().max()) < 1e-3


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("cuts", [[2, 2, 3, 1, 30, 2, 17, 1, 1, 5], [16, 16, 16, 16], [1, 63], [33, 31], [131, 2, 70], [2] * 20])
def test_portions(tmp_path, run, cuts):
    """Portions of several sizes, down to two tokens and one, cut inside and at page borders (pages
    of 16), inside windows and scan chunks: the matrix states carry over every cut."""
    cfg = settle(make_config(), run)
    P = make_checkpoint(tmp_path / "m", cfg, seed=4)
    e = engine_for(tmp_path / "m", run)
    t = toks(sum(cuts), cfg["vocab"], 4)
    want = O.forward(cfg, P, t)
    out, at = [], 0
    for n in cuts:
        out.append(e.step([("a", t[at:at + n], list(range(n)))]))
        at += n
    close(torch.cat(out), want, run, f"portions {cuts}")


@pytest.mark.parametrize("run", RUNS)
def test_mixed_batch_equals_each_alone_and_slots_are_reused(tmp_path, run):
    """Unequal requests in one batch (portions beside single tokens, requests paused for a step),
    a pool of four state slots and few pages, so both are freed and used again: a request that
    takes a used slot starts from zero matrix states."""
    cfg = settle(make_config(), run)
    P = make_checkpoint(tmp_path / "m", cfg, seed=5)
    e = engine_for(tmp_path / "m", run, tokens=240, slots=4)
    V = cfg["vocab"]
    reqs = {k: toks(n, V, 10 + i) for i, (k, n) in enumerate([("a", 120), ("b", 7), ("c", 33), ("d", 1), ("e", 41), ("f", 20)])}
    want = {k: O.forward(cfg, P, v) for k, v in reqs.items()}
    got = {k: [] for k in reqs}
    at = {k: 0 for k in reqs}
    plan = [[("a", 20), ("b", 7)], [("a", 1), ("c", 30), ("d", 1)], [("a", 2), ("c", 1)], [("c", 2), ("a", 97), ("e", 3)],
            [("e", 38), ("f", 5)], [("f", 1)], [("f", 14)]]
    for step in plan:
        entries, end = [], []
        for k, n in step:
            entries.append((k, reqs[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == len(reqs[k]):
                end.append(k)
        out = e.step(entries, end=end)
        o = 0
        for k, n in step:
            got[k].append(out[o:o + n])
            o += n
    for k in reqs:
        close(torch.cat(got[k]), want[k], run, f"request {k}")
    assert e.kv.alloc.num_free == e.kv.num_blocks and len(e.kv.state.free) == 4
    with pytest.raises(KVCacheOOM):       # a fifth live request has no slot
        for i in range(5):
            e.step([(f"x{i}", [1, 2], [])])


@pytest.mark.parametrize("run", RUNS)
def test_long_decoding_past_windows_and_page_borders(tmp_path, run):
    """150 tokens, all but five decoded one by one through pages of 8: every window slides over
    decoded tokens many times. Two sequences decoded together."""
    cfg = settle(make_config(), run)
    P = make_checkpoint(tmp_path / "m", cfg, seed=7)
    e = engine_for(tmp_path / "m", run, block_size=8)
    t, u = toks(150, cfg["vocab"], 7), toks(150, cfg["vocab"], 8)
    out = [e.step([("a", t[:5], list(range(5))), ("b", u[:5], list(range(5)))])]
    a, b = [out[0][:5]], [out[0][5:]]
    for x, y in zip(t[5:], u[5:]):
        o = e.step([("a", [x], [0]), ("b", [y], [0])])
        a.append(o[:1])
        b.append(o[1:])
    close(torch.cat(a), O.forward(cfg, P, t), run, "long decode")
    close(torch.cat(b), O.forward(cfg, P, u), run, "long decode, second sequence")


# ---- the engine's own generation path and scheduler -----------------------------------------------

def _greedy_oracle(P, cfg, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(O.forward(cfg, P, seq)[-1].argmax()))
    return seq[len(prompt):]


@pytest.mark.parametrize("run,graphs", [(("cpu", "fp32"), False), pytest.param(("cuda:0", "fp32"), False, marks=GPU),
                                        pytest.param(("cuda:0", "fp32"), True, marks=GPU)])
def test_greedy_generation_through_run_turns(tmp_path, run, graphs):
    """Greedy decoding through Engine.run_turns (tokenizer, prefix reuse, batched decode loop — the
    captured graph on the GPU) gives the oracle's tokens, for two requests of unequal length, and
    again for a prompt that continues the first reply."""
    cfg = make_config(vocab=300)
    P = make_checkpoint(tmp_path / "m", cfg, seed=8)
    e = engine_for(tmp_path / "m", run, tokens=2048, graphs=graphs)
    sp = SamplingParams(temperature=0.0, max_new_tokens=12, ignore_eos=True, stop_on_consensus=False)
    prompts = ["De ridders aan de ronde tafel overleggen over het cachebeleid.", "Kort."]
    outs = e.run_turns([Turn("A", prompts[0], sp), Turn("B", prompts[1], sp)])
    for o, p in zip(outs, prompts):
        assert o.error is None, o.error
        ids = e.encode_prompt(p)
        assert o.ids == _greedy_oracle(P, cfg, ids, 12)
    from theroundtaible_amd.prompt import Prompt
    p2 = Prompt().add(prompts[0]).add(outs[0].text, outs[0].ids, e.tokenizer.family)
    o2 = e.run_turns([Turn("A", p2, sp)])[0]
    ids2 = e.encode_prompt(prompts[0]) + outs[0].ids
    assert o2.ids == _greedy_oracle(P, cfg, ids2, 12)


@GPU
def test_captured_decode_step_replays_as_eager(tmp_path):
    """The captured decode step, replayed many times with other work between the replays, gives the
    eager loop's tokens: bf16, sizes of the skinny decode GEMM and of the matrix-core attention."""
    layers = [lat(4, 16, 16, 16, 64, window=40, mlp=moe(6, 2, 32, 3, 2)), gla(4, 16, 16, 8.0, moe(6, 2, 32, 3, 2)),
              lat(4, 16, 16, 16, 64, window=24, kv_from=0, mlp=moe(6, 2, 32, 3, 2))]
    cfg = make_config(width=64, vocab=320, layers=layers)
    make_checkpoint(tmp_path / "m", cfg, seed=12)
    sp = SamplingParams(temperature=0.0, max_new_tokens=70, ignore_eos=True, stop_on_consensus=False)
    turns = [Turn("A", "Eerste ridder spreekt over de cache.", sp), Turn("B", "Tweede.", sp), Turn("C", "En de derde ook.", sp)]
    outs = []
    for graphs in (False, True, True):
        e = engine_for(tmp_path / "m", ("cuda:0", "bf16"), tokens=2048, slots=6, graphs=graphs)
        outs.append([o.ids for o in e.run_turns(turns)])
        started = e.start_turns([Turn("D", "Vierde.", sp)])
        seqs, got = [s for s, _, _ in started], [[f] for _, f, _ in started]
        for steps in (3, 9, 20):
            got[0].extend(e.continue_decode(seqs, [Turn("D", "Vierde.", sp)], [got[0][-1]], steps)[0])
            e.step([("x", [1, 2, 3], [])], end=["x"])       # eager work between the replays
            torch.cuda.synchronize()
        outs[-1].append(got[0])
    assert outs[0] == outs[1] == outs[2]


@GPU
def test_decode_steps_on_the_skinny_gemm_and_expert_rows(tmp_path):
    """Sizes the framework's skinny decode GEMM takes (K a multiple of 32, N of 16): decode steps
    run their plain linears on it and their experts row by row; the logits match the oracle and
    the same steps on the library GEMMs."""
    from theroundtaible_amd import ops
    if not ops.native_available():
        pytest.skip("main extension not built")
    layers = [lat(4, 16, 16, 16, 64, window=20, mlp=moe(6, 2, 32, 3, 2)), gla(4, 16, 16, 8.0, moe(6, 2, 32, 3, 2)),
              lat(4, 16, 16, 16, 64, window=9, kv_from=0, mlp=moe(6, 2, 32, 3, 2))]
    cfg = settle(make_config(width=64, vocab=80, layers=layers), ("cuda:0", "bf16"))
    P = make_checkpoint(tmp_path / "m", cfg, seed=11)
    t = toks(60, cfg["vocab"], 11)
    want = O.forward(cfg, P, t)
    outs = []
    for skinny in (True, False):
        e = engine_for(tmp_path / "m", ("cuda:0", "bf16"))
        e.model.use_skinny = skinny
        got = torch.cat([e.step([("a", t[:20], list(range(20)))])] + [e.step([("a", [x], [0])]) for x in t[20:]])
        close(got, want, ("cuda:0", "bf16"), f"skinny={skinny}")
        outs.append(got)
        if skinny:
            assert "w_in" in e.model._dec[0] and all("mix.o" in d for d in e.model._dec.values())
    assert float((outs[0] - outs[1]).abs().max(-1).values.median()) < 0.25


def test_serving_entry_points_match_run_turns():
    """The continuous-batching entry points (prefill + first token, then decode in chunks while the
    state follows) give the tokens of a single run_turns call; random-init preset weights."""
    def eng():
        return Engine(EngineConfig(model="tiny-vurizen", weights="random:3", dtype="fp32", device="cpu",
                                   num_blocks=64, use_graphs=False, state_slots=4))
    sp = SamplingParams(temperature=0.0, max_new_tokens=10, ignore_eos=True, stop_on_consensus=False)
    turns = [Turn("A", "Eerste ridder spreekt over de cache.", sp), Turn("B", "Tweede.", sp)]
    want = [o.ids for o in eng().run_turns(turns)]
    e = eng()
    started = e.start_turns(turns)
    seqs = [s for s, _, _ in started]
    got = [[f] for _, f, _ in started]
    for steps in (4, 5):
        new = e.continue_decode(seqs, turns, [g[-1] for g in got], steps)
        for g, n in zip(got, new):
            g.extend(n)
    assert got == want
    assert all(s.state_len == s.length for s in seqs)


def test_trace_runner_replays_steps(tmp_path):
    """The trace runner's own entry point on the CPU: steps in, logit files out, pages and slots
    given back at the end of a request."""
    import io
    import sys
    import numpy as np
    from theroundtaible_amd import trace_run
    cfg = make_config(vocab=50)
    P = make_checkpoint(tmp_path / "m", cfg, seed=9)
    t = toks(30, 50, 9)
    want = O.forward(cfg, P, t)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": t[:20], "want": [0, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": t[20:22], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": t[22:], "want": [7]}, {"id": "b", "tokens": t[:3], "want": [2]}],
              "end": ["a", "b"]}]
    old_in, old_out = sys.stdin, sys.stdout
    sys.stdin, sys.stdout = io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n"), io.StringIO()
    try:
        rc = trace_run.main(["--model", str(tmp_path / "m"), "--dtype", "float32", "--out", str(tmp_path / "o"),
                             "--max-tokens", "128", "--device", "cpu"])
        said = sys.stdout.getvalue()
    finally:
        sys.stdin, sys.stdout = old_in, old_out
    assert rc == 0 and [l for l in said.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    assert not os.path.exists(tmp_path / "o" / "1.f32")
    a = np.fromfile(tmp_path / "o" / "0.f32", dtype="<f4").reshape(2, 50)
    b = np.fromfile(tmp_path / "o" / "2.f32", dtype="<f4").reshape(2, 50)
    got = torch.tensor(np.concatenate([a, b])).double()
    assert float((got - want[[0, 19, 29, 2]]).abs().max()) < 1e-3
