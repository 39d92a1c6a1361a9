// act(gate) * up of the feed-forwards.
#include "../glu.h"

void gated_mul(torch::Tensor out, torch::Tensor z, int64_t up_at, bool gelu) {
  if (gelu) helix::launch_glu<helix::GeluTanh>(out, z, up_at);
  else helix::launch_glu<helix::Silu>(out, z, up_at);
}
