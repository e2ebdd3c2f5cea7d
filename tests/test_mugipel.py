"""The Mugipel design in the serving engine against the float64 oracle (tests/oracles): small
configurations with random weights written as model folders (config.json + model.safetensors),
loaded through the engine's own registry and driven through its step function (``feed``), its
scheduler (``generate``) and the replay command line.  The CPU runs use the op library's torch
references, the GPU runs (marked) the HIP kernels; both in float32 (sharp) and bfloat16.

Weights are rounded to bfloat16 as stored, so product and oracle see the same numbers.
"""
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

from distributed_llm_amd.engine.llm_engine import BS, LLMEngine
from distributed_llm_amd.engine.sampling import SamplingParams
from oracles import mugipel_oracle as orc

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ----------------------------------------------------------------------------- model folders

def ff(n=20):
    return {"kind": "dense", "ff": n}


def yarn(factor=4.0, original=64, fast=8.0, slow=1.0):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def attn(heads=4, kv_heads=2, dim=8, vdim=6, rot=4, base=100.0, scaling=yarn(), scale=0.4, softcap=3.0, size=9, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": softcap, "mask": {"size": size}}
    if rot:
        m["rot"] = {"dims": rot, "base": base}
        if scaling:
            m["rot"]["scaling"] = dict(scaling)
    return {"type": "attention", "mixer": m, "mlp": mlp}


def latent(heads=3, dim=6, vdim=10, rank=12, scale=0.4, mlp=None):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "scale": scale}, "mlp": mlp}


def make_cfg(layers, loop=None, width=24, vocab=40, eps=1e-5, mult=0.6):
    cfg = {"architecture": "Mugipel", "norm": {"eps": eps}, "residual_mult": mult, "vocab": vocab, "width": width,
           "layers": json.loads(json.dumps(layers))}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def make_weights(cfg, seed=0, qk_gain=1.0, sink=1.0):
    g = torch.Generator().manual_seed(seed)
    W, wd = {}, cfg["width"]
    r = lambda *s, k=1.0: torch.randn(*s, generator=g) * k
    lin = lambda o, i, k=1.0: r(o, i, k=k / math.sqrt(i))
    W["embed"], W["final.norm"] = r(cfg["vocab"], wd), 0.2 * r(wd)
    if "loop" in cfg:
        W["loop.in"], W["loop.step"] = lin(wd, 2 * wd), 0.5 * r(cfg["loop"]["times"], wd)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        W[p + "norm1"] = 0.3 * r(wd) - 0.1
        W[p + "mix.q"], W[p + "mix.g"], W[p + "mix.o"] = lin(H * d, wd, qk_gain), lin(H * dv, wd, 1.5), lin(wd, H * dv)
        if L["type"] == "attention":
            G = m["kv_heads"]
            W[p + "mix.k"], W[p + "mix.v"] = lin(G * d, wd, qk_gain), lin(G * dv, wd)
            W[p + "mix.sink"] = sink + 0.5 * r(H)
        else:
            W[p + "mix.dkv"], W[p + "mix.dkv.norm"] = lin(m["kv_rank"], wd), 1 + 0.3 * r(m["kv_rank"])
            W[p + "mix.uk"], W[p + "mix.uv"] = lin(H * d, m["kv_rank"], qk_gain), lin(H * dv, m["kv_rank"])
        if L.get("mlp"):
            n = L["mlp"]["ff"]
            W[p + "mlp.up"], W[p + "mlp.down"] = lin(n, wd), lin(wd, n)
    return {k: v.to(torch.bfloat16).contiguous() for k, v in W.items()}


def write_model(path, cfg, W):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(W, os.path.join(path, "model.safetensors"))
    return str(path)


def engine(path, device, dtype, rows=3, tokens=256, prefix_cache=False):
    return LLMEngine(path, device=device, dtype=dtype, max_num_seqs=rows, max_model_len=tokens,
                     num_kv_blocks=(tokens + BS - 1) // BS, prefix_cache=prefix_cache)


def close(got, want, dtype, what=""):
    """Row-wise error after removing the mean, relative to the logits' spread."""
    want = want.to(torch.float32)
    d = got.float() - want
    d = d - d.mean(-1, keepdim=True)
    spread = (want - want.mean(-1, keepdim=True)).pow(2).mean().sqrt()
    rows = d.pow(2).mean(-1).sqrt() / spread
    limit = 3e-4 if dtype == torch.float32 else 0.12      # bfloat16: rounding at these widths gives 0.01 to 0.05
    assert float(rows.max()) < limit, f"{what}: relative error {float(rows.max()):.3g} at row {int(rows.argmax())}"


# a loop with an attention layer at its start; sizes differ from layer to layer
FULL = [attn(mlp=ff()), latent(mlp=ff(28)), attn(heads=6, kv_heads=3, dim=6, vdim=10, rot=6, scaling=None, size=21, softcap=5.0, mlp=ff()),
        latent(heads=5, dim=4, vdim=4, rank=8), attn(heads=3, kv_heads=1, dim=10, vdim=5, rot=2, size=64, scale=0.6)]
FULL_LOOP = (2, 4, 3)

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]


def toks(n, vocab=40, seed=0):
    g = torch.Generator().manual_seed(100 + seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


@pytest.fixture(scope="module")
def full_model(tmp_path_factory):
    cfg = make_cfg(FULL, FULL_LOOP)
    W = make_weights(cfg, seed=1)
    return write_model(tmp_path_factory.mktemp("full"), cfg, W), cfg, W


_WANT = {}


def full_want(full_model, t):
    key = tuple(t)
    if key not in _WANT:
        _WANT[key] = orc.forward(t, full_model[2], full_model[1])
    return _WANT[key]


# ----------------------------------------------------------------------------- each mechanism alone

SINGLE = {
    "attention": ([attn()], {}), "attention-with-ff": ([attn(mlp=ff(31))], {}),
    "attention-ungrouped": ([attn(heads=3, kv_heads=3, dim=5, vdim=9, rot=2, size=4)], {}),
    "attention-one-kv-head": ([attn(heads=4, kv_heads=1, dim=6, vdim=4, rot=6, size=30)], {}),
    "attention-no-rot": ([attn(rot=0)], {}), "attention-no-scaling": ([attn(scaling=None)], {}),
    "attention-yarn-factor-one": ([attn(scaling=yarn(factor=1.0))], {}),
    "attention-yarn-all-divided": ([attn(rot=8, scaling=yarn(factor=8.0, original=3))], {}),
    "attention-yarn-none-divided": ([attn(rot=8, scaling=yarn(factor=8.0, original=1 << 22))], {}),
    "attention-yarn-wide": ([attn(heads=2, kv_heads=1, dim=72, rot=64, base=5e4, scaling=yarn(2.0, 256, 32.0, 1.0), size=60)], {}),
    "attention-chunk-one": ([attn(size=1)], {}), "attention-chunk-two": ([attn(size=2)], {}),
    "attention-one-chunk": ([attn(size=1000)], {}), "attention-no-cap": ([attn(softcap=None)], {}),
    "attention-tight-cap": ([attn(softcap=0.5, scale=2.0)], {}),
    "attention-wide-heads": ([attn(heads=2, kv_heads=1, dim=72, vdim=130, rot=40)], {}),
    "attention-many-heads": ([attn(heads=36, kv_heads=2, dim=4, vdim=3, rot=2)], {}),
    "latent": ([latent()], {}), "latent-with-ff": ([latent(mlp=ff(7))], {}), "latent-one-head": ([latent(heads=1, dim=9, vdim=3, rank=5)], {}),
    "latent-many-heads": ([latent(heads=20, dim=4, vdim=8, rank=16)], {}), "latent-wide": ([latent(heads=2, dim=40, vdim=72, rank=136)], {}),
    "loop-all": ([attn(mlp=ff()), latent()], {"loop": (0, 2, 2)}), "loop-once": ([attn(), latent()], {"loop": (1, 2, 1)}),
    "loop-one-layer": ([latent(), attn(mlp=ff())], {"loop": (1, 2, 4)}), "loop-first": ([attn(), latent(mlp=ff())], {"loop": (0, 1, 3)}),
    "no-multiplier": ([attn(mlp=ff()), latent()], {"mult": 1.0}), "large-eps": ([attn(mlp=ff()), latent()], {"eps": 0.3}),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(SINGLE))
def test_mechanism_alone(tmp_path, device, dtype, name):
    layers, kw = SINGLE[name]
    cfg = make_cfg(layers, **kw)
    W = make_weights(cfg, seed=3)
    eng = engine(write_model(tmp_path / "m", cfg, W), device, dtype)
    t = toks(37)
    want = orc.forward(t, W, cfg)
    got = [eng.feed([("a", t[:31], list(range(31)))])] + [eng.feed([("a", t[i:i + 1], [0])]) for i in range(31, 37)]
    close(torch.cat(got), want, dtype, name)


def test_layer_stream_matches(full_model):
    """The stream after every layer run (a looped layer counts each time), not only the logits."""
    path, cfg, W = full_model
    eng = engine(path, "cpu", torch.float32)
    t = toks(29, seed=7)
    taps = []
    orc.forward(t, W, cfg, taps)
    eng.model.tap = []
    eng.feed([("a", t, [0])], ["a"])
    assert len(eng.model.tap) == len(taps) == 9
    for i, (a, b) in enumerate(zip(eng.model.tap, taps)):
        assert torch.allclose(a.double(), b, atol=3e-4, rtol=1e-4), f"run {i}"


@pytest.mark.parametrize("rot", [{"dims": 64, "base": 1e4, "scaling": yarn(2.0, 256, 32.0, 1.0)},
                                 {"dims": 6, "base": 5000.0, "scaling": yarn(16.0, 4096, 4.0, 2.0)},
                                 {"dims": 8, "base": 100.0, "scaling": yarn(8.0, 64, 3.0, 3.0)}, {"dims": 10, "base": 300.0}])
def test_rotation_table(rot):
    """Frequencies and the factor on cos and sin; fast == slow makes the ramp a step (or a narrow one)."""
    from distributed_llm_amd.models.configs import YarnSpec
    from distributed_llm_amd.ops import rope_cos_sin
    sc = rot.get("scaling")
    spec = YarnSpec(sc["factor"], sc["original"], sc["fast"], sc["slow"]).as_scaling() if sc else None
    tab = rope_cos_sin(3000, rot["dims"], rot["base"], "cpu", spec)
    f, mul = orc.frequencies(rot)
    a = torch.arange(3000, dtype=torch.float64)[:, None] * torch.tensor(f, dtype=torch.float64)
    assert torch.allclose(tab.double(), torch.cat([a.cos(), a.sin()], 1) * mul, atol=1e-6)
    if sc:
        plain, _ = orc.frequencies({"dims": rot["dims"], "base": rot["base"]})
        assert mul > 1.0 and f != plain


# ----------------------------------------------------------------------------- cutting the prompt

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", [[50], [1] * 50, [2] * 25, [17, 2, 15, 1, 1, 3, 11], [16, 16, 16, 2], [9, 9, 9, 9, 9, 5], [3, 47], [49, 1]])
def test_portions_and_decoding(full_model, device, dtype, cuts):
    if device == "cpu" and dtype == torch.bfloat16 and len(cuts) > 8:
        pytest.skip("bfloat16 matrix products on the CPU are slow; the GPU run covers this case")
    eng = engine(full_model[0], device, dtype)
    t = toks(50, seed=1)
    got, at = [], 0
    for n in cuts:
        got.append(eng.feed([("r", t[at:at + n], list(range(n)))], ["r"] if at + n == len(t) else []))
        at += n
    close(torch.cat(got), full_want(full_model, t), dtype, f"cuts {cuts[:4]}")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens_and_long_decoding(full_model, device, dtype):
    """Positions 0, 1, 2 on their own, then 150 single-token steps past several page borders and
    every layer's chunk borders."""
    if device == "cpu" and dtype == torch.bfloat16:
        pytest.skip("bfloat16 matrix products on the CPU are slow; the GPU run covers this case")
    eng = engine(full_model[0], device, dtype)
    t = toks(153, seed=2)
    want = full_want(full_model, t)
    got = [eng.feed([("r", t[i:i + 1], [0])]) for i in range(len(t))]
    close(torch.cat(got[:3]), want[:3], dtype, "first tokens")
    close(torch.cat(got), want, dtype, "long decoding")
    for n in (1, 2):      # a whole request of one and of two tokens
        close(eng.feed([("s", t[:n], list(range(n)))], ["s"]), want[:n], dtype, f"{n}-token request")


# ----------------------------------------------------------------------------- batches, rows, pages

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("expand_min", [1, 10 ** 9])      # latent layers: keys and values of every portion made from latents, or never
def test_mixed_batches_and_reuse(full_model, monkeypatch, device, dtype, expand_min):
    """Unequal requests share steps (portions beside single tokens); more requests than batch rows
    and more tokens than pages pass through, so rows and pages are used again."""
    from distributed_llm_amd.ops import seqmix
    monkeypatch.setattr(seqmix, "LATENT_EXPAND_MIN", expand_min)
    eng = engine(full_model[0], device, dtype, rows=3, tokens=112)       # 7 pages of 16
    lens = [40, 9, 33, 1, 21, 30, 5]
    reqs = {f"q{i}": toks(n, seed=10 + i) for i, n in enumerate(lens)}
    at = {k: 0 for k in reqs}
    got = {k: [] for k in reqs}
    waiting, live = list(reqs), []
    pattern, step = [7, 1, 2, 1, 16, 1, 3, 1], 0
    while waiting or live:
        used = sum((len(reqs[k]) + BS - 1) // BS for k in live)
        while waiting and len(live) < 3 and used + (len(reqs[waiting[0]]) + BS - 1) // BS <= 7:
            used += (len(reqs[waiting[0]]) + BS - 1) // BS
            live.append(waiting.pop(0))
        entries, end = [], []
        for j, k in enumerate(live):
            if step % 5 == 3 and j == 1:      # a live request left out of the step
                continue
            n = min(pattern[(step + 3 * j) % len(pattern)], len(reqs[k]) - at[k])
            entries.append((k, reqs[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == len(reqs[k]):
                end.append(k)
        out = eng.feed(entries, end)
        o = 0
        for k, tk, _ in entries:
            got[k].append(out[o:o + len(tk)])
            o += len(tk)
        live = [k for k in live if k not in end]
        step += 1
    for k in reqs:
        close(torch.cat(got[k]), full_want(full_model, reqs[k]), dtype, k)
    assert eng.bm.num_free_blocks() == 7 and len(eng._free_rows) == 3


# ----------------------------------------------------------------------------- chunk edges, far keys, the sink

def _needle(cfg, W, n, pos_a, pos_b, fill=0):
    """The token whose place (position ``pos_a`` instead of ``pos_b``) moves the oracle's last logits
    most, and that movement relative to the logits' spread."""
    best = (0.0, 1)
    for tok in range(1, 12):
        a, b = [fill] * n, [fill] * n
        a[pos_a], b[pos_b] = tok, tok
        la, lb = orc.forward(a, W, cfg)[-1], orc.forward(b, W, cfg)[-1]
        best = max(best, (float((la - lb).std() / la.std()), tok))
    return best


def _prompt_decode_cut(eng, t, cut, what, want):
    """The whole prompt in one step; then cut at ``cut``, the rest as a portion, the last token alone."""
    n = len(t)
    close(eng.feed([("w", t, list(range(n)))], ["w"]), want, torch.float32, f"prompt, {what}")
    got = [eng.feed([("c", t[:cut], list(range(cut)))])] if cut else []
    if n - 1 > cut:
        got.append(eng.feed([("c", t[cut:n - 1], list(range(n - 1 - cut)))]))
    got.append(eng.feed([("c", t[n - 1:], [0])], ["c"]))
    close(torch.cat(got), want, torch.float32, f"cut and decoded, {what}")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size,n", [(2, 42), (15, 45), (16, 48), (17, 60), (63, 126), (64, 100), (65, 131), (100, 130)])
def test_chunk_edges(tmp_path, device, size, n):
    """A prompt of one repeated token with one other token placed on the first position of the last
    position's chunk (seen) or just before it (not seen), chosen and scaled so that the row's weight
    lies on it: a chunk that is one key off moves the logits by about their spread.  Chunks count from
    position 0 of the sequence wherever the prompt is cut."""
    cfg = make_cfg([attn(heads=2, kv_heads=1, dim=8, vdim=5, rot=4, scale=3.0, softcap=20.0, size=size)], width=16)
    first = (n - 1) // size * size
    for seed in range(size, size + 500, 100):      # the first weights that show the edge
        W = make_weights(cfg, seed=seed, qk_gain=2.0)
        move, tok = _needle(cfg, W, n, first, first - 1)
        if move > 0.1:
            break
    assert move > 0.1, "the test's weights do not show the edge"
    eng = engine(write_model(tmp_path / "m", cfg, W), device, torch.float32)
    for at in (first - 1, first, min(first + 1, n - 2)):
        t = [0] * n
        t[at] = tok
        _prompt_decode_cut(eng, t, at, f"other token at {at} of {n}", orc.forward(t, W, cfg))
    # the chunk's first token decoded alone, and a cut inside the chunk
    t = [0] * n
    t[first] = tok
    want = orc.forward(t, W, cfg)
    got = [eng.feed([("d", t[:first], list(range(first)))])] + [eng.feed([("d", t[i:i + 1], [0])]) for i in range(first, n)]
    close(torch.cat(got), want, torch.float32, "chunk decoded from its first token")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("expand_min", [1, 10 ** 9])
@pytest.mark.parametrize("n", [15, 16, 17, 63, 64, 65, 130, 330])
def test_far_keys_of_the_latent_attention(tmp_path, monkeypatch, device, n, expand_min):
    """A softmax so sharp that one key, far back among repeated ones and on either side of a page (16)
    or key-tile (32, 64) border, carries a row; prompts and decoded rows."""
    from distributed_llm_amd.ops import seqmix
    monkeypatch.setattr(seqmix, "LATENT_EXPAND_MIN", expand_min)
    cfg = make_cfg([latent(heads=2, dim=8, vdim=5, rank=10, scale=2.0)], width=16)
    for seed in range(n, n + 500, 100):
        W = make_weights(cfg, seed=seed, qk_gain=2.0)
        moves = []
        for tok in range(1, 12):
            t = [0] * n
            a = orc.forward(t, W, cfg)[-1]
            t[1] = tok
            moves.append((float((orc.forward(t, W, cfg)[-1] - a).std() / a.std()), tok))
        move, tok = max(moves)
        if move > 0.1:
            break
    assert move > 0.1, "the test's weights do not show the far key"
    eng = engine(write_model(tmp_path / "m", cfg, W), device, torch.float32, tokens=512)
    for at in sorted({1, n // 2, n - 2}):
        t = [0] * n
        t[at] = tok
        _prompt_decode_cut(eng, t, at, f"other token at {at} of {n}", orc.forward(t, W, cfg))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("sink", [-6.0, 0.0, 4.0, 30.0])
def test_the_sink_takes_weight(tmp_path, device, sink):
    """The sink's score against scores that the cap keeps small: from no share of a row's denominator
    to nearly all of it; neither scaled nor capped."""
    cfg = make_cfg([attn(scale=0.2, softcap=2.0, size=40)], width=16)
    W = make_weights(cfg, seed=2, sink=sink)
    t = toks(30, seed=3)
    want = orc.forward(t, W, cfg)
    W0 = dict(W)
    W0["l0.mix.sink"] = W["l0.mix.sink"] - 40.0      # next to no sink
    without = orc.forward(t, W0, cfg)
    assert (float((want - without).std() / want.std()) > 0.03) == (sink > -6.0), "the test's sink does not show"
    eng = engine(write_model(tmp_path / "m", cfg, W), device, torch.float32)
    close(eng.feed([("a", t, list(range(30)))], ["a"]), want, torch.float32, f"sink {sink}")


@pytest.mark.parametrize("device", DEVICES)
def test_passes_have_caches_of_their_own(tmp_path, device):
    """Cut prompts through a looped latent layer with sharp scores: a pass that read another pass's
    pages (the same inside one step's prompt, stale or overwritten across steps) would show."""
    cfg = make_cfg([latent(heads=2, dim=8, vdim=8, rank=12, scale=1.5), attn(size=40)], loop=(0, 1, 3), width=16)
    W = make_weights(cfg, seed=5, qk_gain=2.0)
    t = toks(40, seed=4)
    want = orc.forward(t, W, cfg)
    eng = engine(write_model(tmp_path / "m", cfg, W), device, torch.float32)
    assert len(eng.kv_caches) == 4 and len({c[0].data_ptr() for c in eng.kv_caches}) == 4
    got, at = [], 0
    for n in [5, 1, 2, 1, 20, 1, 3, 7]:
        got.append(eng.feed([("t", t[at:at + n], list(range(n)))]))
        at += n
    close(torch.cat(got), want, torch.float32, "looped latent layer, cut")


# ----------------------------------------------------------------------------- the engine's own entry points

def greedy_ok(prompt, out, W, cfg, n):
    """Every generated token is the oracle's arg-max after the tokens before it (the sampler reads
    logits rounded to bfloat16, so a token within that rounding of the best counts)."""
    assert len(out) == n
    lg = orc.forward(prompt + out[:-1], W, cfg)[len(prompt) - 1:]
    for row, t in zip(lg, out):
        top = float(row.max())
        assert float(row[t]) >= top - abs(top) * 2.0 ** -7, (t, int(row.argmax()))



@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("prefix_cache", [False, True])
def test_greedy_generation(full_model, device, prefix_cache):
    """``generate`` (scheduler, admission, prefill, decode steps, sampler) continues prompts as the
    oracle's arg-max does; more prompts than batch rows, so rows turn over; with the prefix cache,
    prompts that share whole pages."""
    path, cfg, W = full_model
    eng = engine(path, device, torch.float32, rows=2, prefix_cache=prefix_cache)
    prompts = [toks(n, seed=20 + n) for n in (5, 23, 1, 12)]
    if prefix_cache:
        base = toks(40, seed=60)
        prompts = [base, base[:33] + toks(4, seed=61), base, base[:17]]
    outs = eng.generate(prompts[:2], SamplingParams(max_new_tokens=8, temperature=0.0, ignore_eos=True))
    outs += eng.generate(prompts[2:], SamplingParams(max_new_tokens=8, temperature=0.0, ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert o.error is None
        greedy_ok(p, o.token_ids, W, cfg, 8)
    # the sampler on this model's logits
    sp = SamplingParams(max_new_tokens=6, temperature=0.9, top_p=0.9, top_k=20, ignore_eos=True)
    for o in eng.generate(prompts[:2], sp):
        assert o.error is None and len(o.token_ids) == 6 and all(0 <= x < cfg["vocab"] for x in o.token_ids)


def test_replay_command_line(full_model, tmp_path):
    """bin/trace_run on a model folder: steps from standard input, logits files, ``done`` lines."""
    path, cfg, W = full_model
    a, b = toks(21, seed=1), toks(6, seed=2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:18], "want": [0, 17]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[18:19], "want": []}, {"id": "b", "tokens": b, "want": [5]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[19:], "want": [1]}], "end": ["a"]}]
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "64", "--device", "cpu"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    wa, wb = orc.forward(a, W, cfg), orc.forward(b, W, cfg)
    read = lambda k, n: torch.from_numpy(np.fromfile(out / f"{k}.f32", dtype="<f4").reshape(n, -1))
    close(read(0, 2), wa[[0, 17]], torch.float32, "step 0")
    close(read(1, 1), wb[[5]], torch.float32, "step 1")
    close(read(2, 1), wa[[20]], torch.float32, "step 2")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_unaligned_sizes(tmp_path, device, dtype):
    """Width, vocabulary and head sizes that no 16-byte vector or 64-wide tile divides: every kernel's
    scalar tail and the library-GEMM routes; generation samples from an unaligned vocabulary."""
    layers = [attn(heads=5, kv_heads=5, dim=6, vdim=7, rot=2, size=11, mlp=ff(9)), latent(heads=3, dim=5, vdim=3, rank=7, mlp=ff(11)),
              latent(heads=7, dim=3, vdim=9, rank=10), attn(heads=3, kv_heads=1, dim=10, vdim=3, rot=10, size=7)]
    cfg = make_cfg(layers, loop=(1, 3, 2), width=20, vocab=37)
    W = make_weights(cfg, seed=6)
    eng = engine(write_model(tmp_path / "m", cfg, W), device, dtype)
    t = toks(30, vocab=37, seed=3)
    want = orc.forward(t, W, cfg)
    got = [eng.feed([("a", t[:21], list(range(21)))])] + [eng.feed([("a", t[i:i + 1], [0])]) for i in range(21, 30)]
    close(torch.cat(got), want, dtype, "unaligned")
    if dtype == torch.float32:
        out = eng.generate([t[:7]], SamplingParams(max_new_tokens=5, temperature=0.0, ignore_eos=True))[0]
        greedy_ok(t[:7], out.token_ids, W, cfg, 5)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("expand_min", [1, 32, 10 ** 9])
def test_aligned_sizes_take_the_matrix_core_paths(tmp_path, monkeypatch, dtype, expand_min):
    """Sizes that the matrix-core kernels and the tuned GEMMs take (bf16), against the oracle; prompt
    portions, decoding and mixed steps; chunks that leave whole key tiles out."""
    from distributed_llm_amd.ops import seqmix
    monkeypatch.setattr(seqmix, "LATENT_EXPAND_MIN", expand_min)
    layers = [attn(heads=4, kv_heads=2, dim=32, vdim=64, rot=16, size=40, mlp=ff(128)), latent(heads=4, dim=32, vdim=64, rank=64, mlp=ff(64)),
              attn(heads=8, kv_heads=1, dim=48, vdim=40, rot=48, size=130, mlp=ff(64)), latent(heads=2, dim=64, vdim=32, rank=160),
              attn(heads=2, kv_heads=2, dim=128, vdim=96, rot=64, size=7)]
    cfg = make_cfg(layers, loop=(1, 4, 2), width=128, vocab=64)
    W = make_weights(cfg, seed=8)
    eng = engine(write_model(tmp_path / "m", cfg, W), "cuda", dtype, tokens=512)
    a, b = toks(250, vocab=64, seed=1), toks(90, vocab=64, seed=2)
    wa, wb = orc.forward(a, W, cfg), orc.forward(b, W, cfg)
    ga = [eng.feed([("a", a[:200], list(range(200)))])]
    out = eng.feed([("a", a[200:201], [0]), ("b", b[:70], list(range(70)))])
    ga.append(out[:1])
    gb = [out[1:]]
    for i in range(20):
        out = eng.feed([("a", a[201 + i:202 + i], [0]), ("b", b[70 + i:71 + i], [0])])
        ga.append(out[:1])
        gb.append(out[1:])
    ga.append(eng.feed([("a", a[221:], list(range(29)))], ["a"]))
    close(torch.cat(ga), wa, dtype, "a")
    close(torch.cat(gb), wb, dtype, "b")


def test_registry_reads_config(full_model):
    from distributed_llm_amd.models.configs import DenseSpec, HybridConfig, LoopSpec, YarnSpec, config_from_dir, mugipel_config
    path, cfg, W = full_model
    c = config_from_dir(path)
    assert isinstance(c, HybridConfig) and c.family == "mugipel" and c.n_layers == len(cfg["layers"])
    assert c.pre_norm and not c.post_norm and c.parallel_ff and c.norm_offset and c.tied_head and c.residual_mult == 0.6
    assert c.loop == LoopSpec(2, 4, 3) and [i for i, _ in c.runs] == [0, 1, 2, 3, 2, 3, 2, 3, 4]
    assert [t for _, t in c.runs] == [None, None, 0, None, 1, None, 2, None, None]
    m = c.layers[0].mixer
    assert m.kind == "gated_attention" and m.paged and not m.recurrent and (m.chunk, m.softcap, m.scale) == (9, 3.0, 0.4)
    assert m.rot.yarn == YarnSpec(4.0, 64.0, 8.0, 1.0) and c.layers[2].mixer.rot.yarn is None
    m = c.layers[1].mixer
    assert m.kind == "latent_attention" and m.gate and (m.q_rank, m.rot_dim, m.kv_rank) == (0, 0, 12)
    assert isinstance(c.layers[0].mlp, DenseSpec) and c.layers[0].mlp.act == "relu2" and c.layers[3].mlp is None
    assert c.num_params() == sum(v.numel() for v in W.values())
    for bad_loop in ((2, 2, 1), (0, 6, 1), (0, 2, 0)):
        bad = json.loads(json.dumps(cfg))
        bad["loop"] = dict(zip(("start", "stop", "times"), bad_loop))
        with pytest.raises(ValueError):
            mugipel_config(bad)
    bad = json.loads(json.dumps(cfg))
    bad["layers"][0]["mixer"]["kv_heads"] = 3
    with pytest.raises(ValueError):
        mugipel_config(bad)


@pytest.mark.parametrize("device", DEVICES)
def test_random_weights(device):
    """The seeded random tensors that benchmarks use have the checkpoint's names and sizes."""
    from distributed_llm_amd.models.configs import mugipel_config
    from distributed_llm_amd.models.registry import build_model
    cfg = mugipel_config(make_cfg(FULL, FULL_LOOP))
    m = build_model(cfg, device=device, dtype=torch.float32)
    names = m._random(0, 0.02)
    assert sum(v.numel() for v in names.values()) == cfg.num_params()
    twice = sum(L["uv"].numel() for L in m.layers if "uv" in L)      # the value up-projections are kept in two layouts
    assert m.weight_bytes() == 4 * (cfg.num_params() + twice) and m.decode_read_bytes() > m.weight_bytes()
