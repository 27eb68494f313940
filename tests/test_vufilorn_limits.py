"""What Vufilorn does not have is refused with a clear error, not run wrongly."""
import pytest
import torch

from distributed_llm_alignment_amd.models import build_model, generate, get_config


def test_parallel_forms_and_fp8_are_refused():
    from distributed_llm_alignment_amd.parallel.layer_split import dispatch_layers
    from distributed_llm_alignment_amd.parallel.tensor_parallel import apply_tensor_parallel

    m = build_model(get_config("tiny-vufilorn"), device="cpu", seed=0)
    with pytest.raises(NotImplementedError):
        apply_tensor_parallel(m, None, tp_rank=0, tp_size=2)
    with pytest.raises(NotImplementedError):
        dispatch_layers(m, ["cpu", "cpu"])
    with pytest.raises(ValueError):
        generate(m, torch.zeros(1, 3, dtype=torch.long), max_new_tokens=2, weight_dtype="fp8")


def test_bench_serve_option_and_peer():
    import bench
    from distributed_llm_alignment_amd.eval import serve_bench

    a = bench.parse([])
    assert a.serve is None and a.model == "llama3-8b"  # the default workload is untouched
    assert bench.parse(["--serve"]).serve == "vufilorn"
    cfg = get_config("vufilorn-1b")
    peer = serve_bench.peer_config(cfg, len(cfg.layer_schedule))
    assert peer.hidden_size == cfg.hidden_size and peer.num_layers == len(cfg.layer_schedule)
    assert peer.sliding_window == 4096


def test_eval_latency_runs_the_design():
    from distributed_llm_alignment_amd.eval.eval_latency import measure_model

    m = build_model(get_config("tiny-vufilorn"), device="cpu", seed=0).eval()
    rows = measure_model(m, [2], [12], 1, 1, decode_tokens=3)
    assert rows[0]["decode_tokens_per_second"] > 0


def test_teacher_generation_program(tmp_path):
    """The command line around generate() takes the design by preset name."""
    import json

    from distributed_llm_alignment_amd.training.generate_teacher_data import main

    (tmp_path / "p.jsonl").write_text("".join(json.dumps({"prompt": t}) + "\n" for t in ("a", "some longer prompt")))
    assert main(["--teacher", "tiny-vufilorn", "--prompts", str(tmp_path / "p.jsonl"), "--output", str(tmp_path / "o.jsonl"),
                 "--batch_size", "2", "--max_new_tokens", "5"]) == 0
    assert len((tmp_path / "o.jsonl").read_text().splitlines()) == 2
