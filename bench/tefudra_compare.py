"""Prefill and decode throughput of the Tefudra design beside the closest uniform family (Llama: sequential pre-norm
blocks, RMS norm, rotary grouped-query attention, gated feed-forward) at equal size, random weights, through the serving
engine (scheduler, paged cache, state slots, decode graphs, sampler). Run as ``python bench.py --tefudra [SIZE,...]``.

Tefudra: four layers - pair (attention | matrix memory) + dense, attention + experts, pair + experts, attention + dense.
"Equal size": same width, vocabulary and number of layers, the attention's heads, key/value heads and head size; the dense
family's gated feed-forward holds as many numbers as a Tefudra token touches in an expert layer (ungated: two matrices of top
x expert ff + shared ff; gated: three).
"""
from __future__ import annotations

import torch

from timisun_compare import measure

SIZES = {
    # width; attention heads / key heads / head size / window / kept; pair's window; memory heads x key size x value size;
    # experts / identity / top / expert ff / shared ff; dense ff
    "w1024": dict(width=1024, heads=8, kv=2, dim=128, window=512, keep=4, lwindow=512, mheads=4, mdim=128, mvdim=256,
                  experts=16, ident=4, top=2, eff=768, sff=1536, ff=3072, vocab=32000),
    "w2048": dict(width=2048, heads=16, kv=4, dim=128, window=512, keep=4, lwindow=512, mheads=8, mdim=128, mvdim=256,
                  experts=32, ident=8, top=4, eff=1152, sff=1536, ff=6144, vocab=32000),
    "w4096": dict(width=4096, heads=32, kv=8, dim=128, window=1024, keep=4, lwindow=1024, mheads=16, mdim=128, mvdim=256,
                  experts=64, ident=8, top=4, eff=2304, sff=3072, ff=12288, vocab=32000),
}
LAYERS = 4


def tefudra_dict(s):
    dense = dict(kind="dense", ff=s["ff"])
    moe = dict(kind="moe", router=dict(experts=s["experts"], top=s["top"], identity=s["ident"]),
               expert=dict(ff=s["eff"]), shared=dict(ff=s["sff"]))
    common = dict(heads=s["heads"], kv_heads=s["kv"], dim=s["dim"], vdim=s["dim"], scale=s["dim"] ** -0.5)
    att = dict(**common, mask=dict(size=s["window"], keep_first=s["keep"]), rot=dict(base=500000.0, dims=s["dim"] // 2))
    pair = dict(left=dict(**common, conv=4, softcap=30.0, mask=dict(size=s["lwindow"]), rot=dict(base=10000.0, dims=s["dim"])),
                right=dict(heads=s["mheads"], dim=s["mdim"], vdim=s["mvdim"], gate_cap=15.0))
    return dict(architecture="Tefudra", vocab=s["vocab"], width=s["width"], norm=dict(eps=1e-6, groups=4),
                layers=[dict(type="parallel", mixer=pair, mlp=dense), dict(type="attention", mixer=att, mlp=moe),
                        dict(type="parallel", mixer=pair, mlp=moe), dict(type="attention", mixer=att, mlp=dense)])


def dense_ff(s):
    return (s["top"] * s["eff"] + s["sff"]) * 2 // 3 // 64 * 64


def build(kind, s, dev):
    from llmss_amd.models.config import ModelConfig, get_preset
    from llmss_amd.models.layered import create_model
    from llmss_amd.models.weights import random_tefudra_weights, random_weights

    if kind == "tefudra":
        cfg = ModelConfig.from_hf_dict(tefudra_dict(s))
        return create_model(cfg, random_tefudra_weights(cfg, device=dev, dtype=torch.bfloat16, seed=1))
    cfg = get_preset("llama2-7b", hidden_size=s["width"], num_layers=LAYERS, num_heads=s["heads"],
                     num_kv_heads=s["kv"], head_dim=s["dim"], intermediate_size=dense_ff(s), vocab_size=s["vocab"],
                     max_position_embeddings=8192, rotary_dim=s["dim"])
    return create_model(cfg, random_weights(cfg, device=dev, dtype=torch.bfloat16, seed=1))


def run(sizes, batch, prompt_len, gen_len, rounds, progress, kinds=("tefudra", "dense")):
    dev = torch.device("cuda", torch.cuda.current_device())
    rows = []
    for name in sizes:
        s = SIZES[name]
        row = dict(size=name, shape=s, batch=batch, prompt_len=prompt_len, gen_len=gen_len)
        for kind in kinds:
            progress(f"{name} {kind}: building")
            model = build(kind, s, dev)
            row[kind] = measure(model, batch, prompt_len, gen_len, rounds, progress)
            row[kind]["params_M"] = round(model.cfg.num_params() / 1e6, 1)
            del model
            torch.cuda.empty_cache()
        if "tefudra" in row and "dense" in row:
            row["prefill_ratio"] = round(row["tefudra"]["prefill_tok_s"] / row["dense"]["prefill_tok_s"], 3)
            row["decode_ratio"] = round(row["tefudra"]["decode_tok_s"] / row["dense"]["decode_tok_s"], 3)
        rows.append(row)
    return dict(metric="tefudra_vs_dense_tokens_per_sec", unit="tokens/s", dtype="bf16", data="synthetic",
                sizes=rows)
