// K3 at head dim 256: the vector kernel's instantiations (see paged_decode.hip).
#include "paged_decode_launch.h"

int mv_paged_decode_launch_d256(const DecodeParams &p, const DecodePlan &pl, int batch, int dtype, int flags, hipStream_t stream) {
  MV_DISPATCH_DTYPE(dtype, return (launch_d<Tag, 256>(p, pl, batch, dtype, flags, stream)));
  return MV_OK;
}
