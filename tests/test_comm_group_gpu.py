"""The separate RCCL groups ZeRO-3 gathers and reduces on (``comm.new_group``): their collectives are exact."""
import os

import pytest
import torch

pytestmark = pytest.mark.gpu


def test_new_group_collectives():
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    import hcache_deepspeed_amd as hds
    from hcache_deepspeed_amd import comm as dist
    os.environ.setdefault("MASTER_PORT", "29581")
    hds.init_distributed(verbose=False)
    g = dist.new_group(ranks=list(range(dist.get_world_size())))
    x = torch.arange(1024, device="cuda", dtype=torch.bfloat16)
    out = torch.empty(1024 * dist.get_world_size(), device="cuda", dtype=torch.bfloat16)
    torch.distributed.all_gather_into_tensor(out, x, group=g)
    torch.distributed.all_reduce(x, group=g)
    torch.cuda.synchronize()
    assert torch.equal(out[:1024], torch.arange(1024, device="cuda", dtype=torch.bfloat16))
    assert torch.equal(x, torch.arange(1024, device="cuda", dtype=torch.bfloat16) * dist.get_world_size())
