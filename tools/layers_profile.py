#!/usr/bin/env python3
"""One workload of a layer-list model for rocprofv3, and the per-kernel summary of its trace.

    rocprofv3 --kernel-trace --stats -d OUT -o t -- python3 tools/layers_profile.py 2048 4 prefill 2048
    rocprofv3 ...                                -- python3 tools/layers_profile.py 2048 4 decode 4096 [--gusorax | --llama]
    python3 tools/layers_profile.py --report OUT/t_results.db

decode T: eager fused steps at positions T ... T + 63 (T <= 2: from an empty sequence); prefill T: four passes of a
T-token prompt.  Default: the Gufanex model of bench.py --layers; --gusorax: the Gusorax one; --llama: the llama-family
model of equal weights per token.
"""
import os
import sqlite3
import sys

sys.path.insert(0, os.path.join(os.path.dirname(os.path.abspath(__file__)), ".."))


def report(db: str) -> None:
    rows = sqlite3.connect(db).execute(
        "select name, count(*), avg(end - start) / 1e3, min(end - start) / 1e3, grid_x, grid_y, grid_z from kernels "
        "where name not like '%at::native%' and name not like '%rocclr%' and name not like '%k_st_%' "
        "group by name, grid_x, grid_y, grid_z order by sum(end - start) desc limit 40").fetchall()
    for r in rows:
        print("%-84s n %5d  avg %8.2f us  min %8.2f us  threads %s" % (r[0].replace("void ", "")[:84], r[1], r[2], r[3], r[4:]))


def main() -> None:
    if sys.argv[1] == "--report":
        return report(sys.argv[2])
    import numpy as np

    import bench
    from kuiperllama_amd import binfmt, checkpoint
    from kuiperllama_amd.model import KuiperModel
    width, layers, mode, T = int(sys.argv[1]), int(sys.argv[2]), sys.argv[3], int(sys.argv[4])
    cfg = bench.layers_config(width, layers, arch="Gusorax" if "--gusorax" in sys.argv else "Gufanex")
    if "--llama" in sys.argv:
        elems, head, _ = bench.layers_work(cfg)
        hidden = int(((elems - head) / layers - 4 * width * width) / (3 * width)) // 64 * 64
        m, keep = bench.build_model(binfmt.ModelSpec(width, hidden, layers, width // 128, width // 128, cfg["vocab"], 4352,
                                                     False, name=f"llama-{width}x{layers}"), 0)
    else:
        m = KuiperModel.from_tensors(cfg, checkpoint.safetensors_image(bench.layers_tensors(cfg)), max_seq_len=4352)
    toks = [int(t) for t in np.random.default_rng(1).integers(0, cfg["vocab"], 4096)]
    if mode == "decode":
        n = max(T, 2)
        for _ in range(2):
            print(m.generate(toks[:n], n + 64, exec="fused")[1], "ms")
    else:
        for _ in range(4):
            print(m.time_prefill(toks[:T], 0), "ms")
    m.close()


if __name__ == "__main__":
    main()
