// What a token's id brings to the stream besides the plain embedding:
//   embed_norm : h[t] = w * e / sqrt(mean(e^2) + eps), e the token's row of the embedding table;
//   token_gate : out[t, j] = gelu_tanh(z[t, j]) * table[token_t, col + j], a layer's own slice of a per-token table, gated
//                by a product of the stream (the product back to the stream's width and its norm follow as usual).
// Everything in 32-bit; tables and weights in their stored type.
#include "common.h"

namespace llme {

__device__ __forceinline__ float gelu_tanh(float z) {
    return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// One workgroup a row, which waits in LDS between the two passes. blocked: the table is in the matrix kernels' layout
// ([V / 16][H / 32] blocks of [4][16][8]; V a multiple of 16, H of 32).
template <typename TT, typename TW>
__global__ __launch_bounds__(256) void embed_norm_kernel(const TT* __restrict__ table, const int* __restrict__ tokens,
                                                         const TW* __restrict__ w, float* __restrict__ out, int H, float eps,
                                                         int blocked) {
    extern __shared__ float row[];
    __shared__ float scratch[4];
    const int t = blockIdx.x, id = tokens[t];
    const TT* src = blocked ? table + static_cast<size_t>(id / 16) * 16 * H + (id % 16) * 8 : table + static_cast<size_t>(id) * H;
    float ss = 0.f;
    for (int i = threadIdx.x; i < H; i += 256) {
        const int j = i / 8;
        const float v = to_float(src[blocked ? static_cast<size_t>(j / 4) * 512 + (j % 4) * 128 + i % 8 : static_cast<size_t>(i)]);
        row[i] = v;
        ss = fmaf(v, v, ss);
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch, 4) / static_cast<float>(H) + eps);
    for (int i = threadIdx.x; i < H; i += 256) out[static_cast<size_t>(t) * H + i] = (to_float(w[i]) * row[i]) * inv;
}

template <typename TT, typename TO>
__global__ __launch_bounds__(256) void token_gate_kernel(const float* __restrict__ z, int ld_z, const TT* __restrict__ table, int ld_table,
                                                         int col, const int* __restrict__ tokens, TO* __restrict__ out, int n, size_t total) {
    const size_t i = static_cast<size_t>(blockIdx.x) * 256 + threadIdx.x;
    if (i >= total) return;
    const size_t t = i / n;
    const int j = static_cast<int>(i % n);
    out[i] = from_float<TO>(gelu_tanh(z[t * ld_z + j]) * to_float(table[static_cast<size_t>(tokens[t]) * ld_table + col + j]));
}

}  // namespace llme

using namespace llme;

extern "C" int llme_embed_norm(const void* table, int table_dtype, const int* tokens, const void* w, int w_dtype, float* out, int T, int H,
                               float eps, int blocked, hipStream_t stream) {
    if (T <= 0) return 0;
    if (H <= 0 || H > 15000) return kErrUnsupported;
    if (blocked && (table_dtype != kBF16 || H % 32 != 0)) return kErrUnsupported;
    const size_t lds = static_cast<size_t>(H) * sizeof(float);
#define LLME_EN(TT, TW)                                                                                                     \
    hipLaunchKernelGGL((embed_norm_kernel<TT, TW>), dim3(T), dim3(256), lds, stream, static_cast<const TT*>(table), tokens, \
                       static_cast<const TW*>(w), out, H, eps, blocked)
    switch (table_dtype * 2 + w_dtype) {
        case 0: LLME_EN(float, float); break;
        case 1: LLME_EN(float, bf16); break;
        case 2: LLME_EN(bf16, float); break;
        case 3: LLME_EN(bf16, bf16); break;
        default: return kErrBadArgument;
    }
#undef LLME_EN
    return launch_status();
}

extern "C" int llme_token_gate(const float* z, int ld_z, const void* table, int table_dtype, int ld_table, int col, const int* tokens,
                               void* out, int out_dtype, int T, int n, hipStream_t stream) {
    if (T <= 0 || n <= 0) return 0;
    if (ld_z < n || col < 0 || col + n > ld_table) return kErrBadArgument;
    const size_t total = static_cast<size_t>(T) * n;
    const dim3 grid(static_cast<unsigned>((total + 255) / 256));
#define LLME_TG(TT, TO)                                                                                                           \
    hipLaunchKernelGGL((token_gate_kernel<TT, TO>), grid, dim3(256), 0, stream, z, ld_z, static_cast<const TT*>(table), ld_table, col, \
                       tokens, static_cast<TO*>(out), n, total)
    switch (table_dtype * 2 + out_dtype) {
        case 0: LLME_TG(float, float); break;
        case 1: LLME_TG(float, bf16); break;
        case 2: LLME_TG(bf16, float); break;
        case 3: LLME_TG(bf16, bf16); break;
        default: return kErrBadArgument;
    }
#undef LLME_TG
    return launch_status();
}

LLME_LOAD_ENTRY(token_input)
