// bf16 GEMM instantiations for the GeGLU epilogue (gemm_impl.h; dispatched by gai_gemm in gemm.hip).
#include "gemm_impl.h"

GAI_GEMM_RUN(10)
