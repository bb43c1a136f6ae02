"""Small Modepel models, engines around them and helpers of the schedule tests."""
import torch

from replisense_rfq_amd.engine.engine import LLMEngine
from replisense_rfq_amd.models.config import modepel_from_json
from replisense_rfq_amd.models.modepel import ModepelLM
from replisense_rfq_amd.models.weights import init_modepel_weights, modepel_from_full
from replisense_rfq_amd.utils.config import EngineConfig
from tests.livisun.common import alone, run_schedule, tokens  # noqa: F401  (schedule driver)

from . import oracle


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, identity=0, groups=None, scale=1.0, shared=0):
    r = {"experts": experts, "top": top, "scale": scale}
    if identity:
        r["identity"] = identity
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    f = {"kind": "moe", "expert": {"ff": ff}, "router": r}
    if shared:
        f["shared"] = {"ff": shared}
    return f


def attn(heads, kv_heads, dim, vdim, rot_dims, mlp, scale=0.3, base=900.0, v_mix=True):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                      "v_mix": v_mix, "rot": {"base": base, "dims": rot_dims}}}


def memory(heads, dim, vdim, mlp, cap=7.0):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": mlp}


def config(layers, vocab=71, width=48, eps=1e-5):
    return {"architecture": "Modepel", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps}}


# sizes unlike each other and unlike the usual ones: dim != vdim, heads * vdim != width, odd head
# counts, rot_dims < dim, a memory first, a layer without feed-forward, a layer outside the value
# blend between two inside, mixtures with and without identity, groups and shared expert
SMALL = config([
    memory(3, 12, 20, dense(40)),
    attn(6, 2, 16, 12, 8, moe(5, 3, 24, identity=3, groups=(4, 3), scale=1.4, shared=28)),
    attn(3, 1, 10, 8, 10, None, v_mix=False, base=50.0),
    memory(2, 8, 8, moe(6, 2, 16, groups=(3, 2), scale=0.8), cap=3.0),
    attn(4, 2, 20, 12, 4, moe(4, 4, 20, identity=1), scale=0.45),
    attn(2, 2, 8, 12, 6, dense(33)),
])
# values that happen to be 1, equal or all: one head, one kv head, everything rotated, top 1, one
# group, as many choices as router outputs
ONES = config([attn(1, 1, 16, 16, 16, moe(1, 1, 16, identity=1, groups=(1, 1))), memory(1, 16, 16, None),
               attn(4, 1, 8, 16, 0, moe(2, 3, 8, identity=1, shared=8)), memory(1, 1, 1, dense(1))],
              vocab=50, width=32, eps=1e-3)
# nothing a multiple of 4 (width, head sizes, feed-forward widths, vocabulary)
ODD = config([attn(3, 3, 6, 10, 6, dense(18)), memory(3, 7, 9, moe(5, 2, 11, identity=2, groups=(7, 4), shared=13)),
              attn(5, 5, 14, 6, 10, dense(22), v_mix=False), attn(6, 3, 10, 10, 2, dense(10), scale=0.7)],
             vocab=53, width=37)
# sizes the MFMA tiles cover (bf16 on the GPU); sixteen heads over one key head: decoded rows take
# the heads-as-columns form
WIDE = config([attn(8, 2, 32, 32, 16, dense(64), scale=0.2), memory(3, 32, 80, moe(4, 2, 32, identity=2, shared=32)),
               attn(16, 2, 64, 32, 32, moe(4, 2, 32), scale=0.15), attn(16, 1, 32, 64, 16, None, v_mix=False),
               memory(1, 64, 80, dense(64))],
              width=64, vocab=90)


def build(cfg_dict, device="cpu", dtype=torch.float32, seed=0, full=None, **eng_kw):
    cfg = modepel_from_json(cfg_dict, name="test-modepel")
    w = init_modepel_weights(cfg, device, dtype, seed) if full is None \
        else modepel_from_full(full, cfg, device, dtype)
    model = ModepelLM(cfg, device, weights=w, dtype=dtype)
    kw = dict(model="tiny-modepel", device=str(device), max_num_seqs=4, max_kv_blocks=24,
              max_batched_tokens=512, max_model_len=512, use_graphs=False, grammar=False,
              prefix_cache=False, warm_prefix=False, tune_gemm=False, jump_forward=False,
              dtype="float32" if dtype == torch.float32 else "bfloat16")
    kw.update(eng_kw)
    eng = LLMEngine(EngineConfig(**kw), model=model)
    return eng, w["full"]


def check(got, cfg_dict, full, requests, tol=3e-4):
    """Every produced row against the oracle's logits of that request and position."""
    ref = {n: oracle.forward(cfg_dict, full, t) for n, t in requests.items()}
    assert got, "no logits produced"
    for (n, p), row in got.items():
        r = ref[n][p]
        err = float((row.double() - r).abs().max() / r.abs().max())
        assert err < tol, f"request {n} position {p}: relative error {err:.2e}"
