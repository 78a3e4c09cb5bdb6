"""Bezurax (pooled-block attention beside a generalised delta rule, routed experts) inference CLI.  Same modes
and flags as llama3_2_runner.py, one GPU:

    python examples/inference/run_bezurax.py trace --model_path <model dir> --traced_path out
    python examples/inference/run_bezurax.py generate --traced_path out --prompt_ids 1,2,3
    python examples/inference/run_bezurax.py check_accuracy --model_path <model dir> --traced_path out --prompt_ids 1,2,3
check_accuracy compares greedy tokens with the same model computed in 32-bit.
"""

import os
import sys

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
sys.path.insert(0, os.path.join(os.path.dirname(os.path.abspath(__file__)), "..", ".."))

from llama3_2_runner import main  # noqa: E402

from neuronx_distributed_llama3_2_amd.inference.bezurax import BezuraxRunner  # noqa: E402

if __name__ == "__main__":
    main(runner_cls=BezuraxRunner)
