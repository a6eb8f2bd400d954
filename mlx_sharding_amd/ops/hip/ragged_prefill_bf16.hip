// bf16 instances of the expanded latent attention.
#include "ragged_prefill.h"

// nks: ceil(dq / 32) rounded up to {2, 4, 6, 8}; ndh: vdp / 16 in {2, 4, 8, 16}
extern "C" void launch_latent_attn_long_bf16(const LatentLongArgs* a, int nks,
                                             int ndh, hipStream_t stream) {
#define LP_CASE(K, D) \
  case K * 100 + D: latent_attn_long_go<__bf16, K, D>(*a, stream); break
  switch (nks * 100 + ndh) {
    LP_CASE(2, 2); LP_CASE(2, 4); LP_CASE(2, 8); LP_CASE(2, 16);
    LP_CASE(4, 2); LP_CASE(4, 4); LP_CASE(4, 8); LP_CASE(4, 16);
    LP_CASE(6, 2); LP_CASE(6, 4); LP_CASE(6, 8); LP_CASE(6, 16);
    LP_CASE(8, 2); LP_CASE(8, 4); LP_CASE(8, 8); LP_CASE(8, 16);
    default: break;
  }
#undef LP_CASE
}
