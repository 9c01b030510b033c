// Linear attention with one fixed decay a head (lightning attention). Per request and head a memory S [dim, vdim], 32-bit,
// zero at admission; a token with query q, key k and value v (each the SiLU of the input product's columns) does
//   S <- a S + k v^T;  o = S^T q
// and the heads' reads side by side are divided by their common root mean square, multiplied by a weight and by sigmoid of a
// gate (joined_norm_gate).
//
// Kept per slot: memory [heads, vdim, dim], a column's key channels side by side.
//
// A step in which every request brings one row has a kernel of its own. Otherwise two ways through a request's rows, chosen by
// how many it brings (`chunk_from`: that many or more are chunked). The walk (any sizes, 32-bit throughout; short portions, the
// 32-bit model) takes them one by one, columns side by side. The chunked form (bfloat16 model, long portions) uses that the
// rule is linear in S and that the decay does not depend on the tokens: with t counted from a chunk's start,
//   o_t = a^(t+1) S_start^T q_t + sum_(s <= t) a^(t-s) (q_t . k_s) v_s,    S_end = a^n S_start + sum_s a^(n-1-s) k_s v_s^T,
// three kernels on the matrix cores (v_mfma_f32_16x16x32_bf16):
//   add  : what every chunk adds to an empty memory;
//   carry: chunk by chunk S_start (as two bfloat16 parts), the slot's new memory;
//   read : the rows of half a chunk: the product with S_start and the causal product with the chunk's own keys and values.
// q, k and v enter the products as bfloat16 (outputs of a bfloat16 model's projections and their activation); everything that
// carries a power of the decay (values, scores, the memory) enters as the sum of two bfloat16 parts, sums are 32-bit.
#include "common.h"

namespace llme {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
typedef __attribute__((ext_vector_type(4))) float f32x4;

struct LightningInput {
    const float* p;             // [T, ld]: the input product's rows
    int ld, q_col, k_col, v_col;
    const float* decay;         // [2 heads]: the decays, then their logarithms
    int heads, dim, vdim;
};

__device__ __forceinline__ float silu(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float4 silu4(float4 z) { return float4{silu(z.x), silu(z.y), silu(z.z), silu(z.w)}; }

// ---------------------------------------------------------------------------------------------------------------
// The walk. LPC lanes share a column (lane l holds the R key channels l R ..), a workgroup owns 256 / LPC columns of one head
// of one request. Rows come through LDS in blocks of eight (k, q, the columns' values), the next block asked for while the
// current one is worked through.
constexpr int kWalkRows = 8;

template <int R, int LPC>
__global__ __launch_bounds__(256) void lightning_walk_kernel(LightningInput in, float* __restrict__ memory, const int* __restrict__ q_start,
                                                             const int* __restrict__ slots, float* __restrict__ o, int chunk_from) {
    constexpr int DP = LPC * R, COLS = 256 / LPC;
    constexpr int W = 2 * DP + COLS;                        // floats of a row in LDS
    constexpr int BLOCK = kWalkRows * W;
    constexpr int NF = (BLOCK + 255) / 256;
    __shared__ __align__(16) float lds[2 * BLOCK];
    const int s = blockIdx.z, h = blockIdx.y, col0 = blockIdx.x * COLS;
    const int tid = threadIdx.x, cl = tid / LPC, l = tid % LPC;
    const int col = col0 + cl;
    const bool live = col < in.vdim;
    const int first = q_start[s], last = q_start[s + 1];
    if (first >= last || last - first >= chunk_from) return;        // (the whole workgroup)
    float* M = memory + ((static_cast<size_t>(slots[s]) * in.heads + h) * in.vdim + (live ? col : 0)) * in.dim;
    float m[R];
#pragma unroll
    for (int i = 0; i < R; ++i) m[i] = (live && l * R + i < in.dim) ? M[l * R + i] : 0.f;
    const float decay = in.decay[h];

    int from[NF], row_of[NF];                               // a column of p (the same for every block of rows), or none
#pragma unroll
    for (int i = 0; i < NF; ++i) {
        const int e = tid + 256 * i;
        const int x = e % W;
        row_of[i] = e / W;
        from[i] = -1;
        if (e < BLOCK) {
            if (x < DP) {
                if (x < in.dim) from[i] = in.k_col + h * in.dim + x;
            } else if (x < 2 * DP) {
                if (x - DP < in.dim) from[i] = in.q_col + h * in.dim + x - DP;
            } else if (col0 + x - 2 * DP < in.vdim) {
                from[i] = in.v_col + h * in.vdim + col0 + x - 2 * DP;
            }
        }
    }
    float pre[NF];
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < NF; ++i) {
            const int t = t0 + row_of[i];
            pre[i] = (from[i] >= 0 && t < last) ? in.p[static_cast<size_t>(t) * in.ld + from[i]] : 0.f;
        }
    };
    auto put = [&](int buf) {
#pragma unroll
        for (int i = 0; i < NF; ++i) {
            const int e = tid + 256 * i;
            if (e < BLOCK) lds[buf * BLOCK + e] = silu(pre[i]);
        }
    };
    fetch(first);
    put(0);
    __syncthreads();
    int cur = 0;
    for (int t0 = first; t0 < last; t0 += kWalkRows) {
        const bool more = t0 + kWalkRows < last;
        if (more) fetch(t0 + kWalkRows);
        const int nt = min(kWalkRows, last - t0);
        for (int tt = 0; tt < nt; ++tt) {
            const float* row = lds + cur * BLOCK + tt * W;
            const float v = row[2 * DP + cl];
            float reads[2] = {0.f, 0.f};
#pragma unroll
            for (int i = 0; i < R; i += 2) {
                const float2 k2 = *reinterpret_cast<const float2*>(row + l * R + i);
                const float2 q2 = *reinterpret_cast<const float2*>(row + DP + l * R + i);
                m[i] = fmaf(k2.x, v, decay * m[i]);
                m[i + 1] = fmaf(k2.y, v, decay * m[i + 1]);
                reads[0] = fmaf(m[i], q2.x, reads[0]);
                reads[1] = fmaf(m[i + 1], q2.y, reads[1]);
            }
            const float read = sum_of_lanes<LPC>(reads[0] + reads[1]);
            if (live && l == 0) o[(static_cast<size_t>(t0 + tt) * in.heads + h) * in.vdim + col] = read;
        }
        if (more) {
            put(cur ^ 1);
            __syncthreads();
            cur ^= 1;
        }
    }
#pragma unroll
    for (int i = 0; i < R; ++i)
        if (live && l * R + i < in.dim) M[l * R + i] = m[i];
}

// A step in which every request brings one row (decoding): a workgroup takes the row through 64 columns of one head's memory,
// 16 lanes a column (R key channels each), all four passes' columns asked for together. VEC: channels come in whole pieces of four.
template <int R, bool VEC>
__global__ __launch_bounds__(256) void lightning_single_kernel(LightningInput in, float* __restrict__ memory, const int* __restrict__ slots,
                                                               float* __restrict__ o) {
    constexpr int COLS = 16, U = 4;
    const int t = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * COLS * U, tid = threadIdx.x;
    const int cl = tid >> 4, l = tid & 15, vdim = in.vdim, dim = in.dim;
    const float* row = in.p + static_cast<size_t>(t) * in.ld;
    float* M = memory + (static_cast<size_t>(slots[t]) * in.heads + h) * vdim * dim;
    auto load = [&](const float* src, float (&dst)[R]) {
        if constexpr (VEC) {
#pragma unroll
            for (int i = 0; i < R; i += 4) {
                float4 x{0.f, 0.f, 0.f, 0.f};
                if (l * R + i < dim) x = *reinterpret_cast<const float4*>(src + l * R + i);
                dst[i] = x.x; dst[i + 1] = x.y; dst[i + 2] = x.z; dst[i + 3] = x.w;
            }
        } else {
#pragma unroll
            for (int i = 0; i < R; ++i) dst[i] = l * R + i < dim ? src[l * R + i] : 0.f;
        }
    };
    float m[U][R], vv[U], kk[R], qq[R];
#pragma unroll
    for (int u = 0; u < U; ++u) {
        const int c = c0 + u * COLS + cl;
        vv[u] = 0.f;
        if (c < vdim) {
            load(M + static_cast<size_t>(c) * dim, m[u]);
            vv[u] = row[in.v_col + h * vdim + c];
        }
    }
    load(row + in.k_col + h * dim, kk);
    load(row + in.q_col + h * dim, qq);
    const float decay = in.decay[h];
#pragma unroll
    for (int i = 0; i < R; ++i) {
        kk[i] = silu(kk[i]);
        qq[i] = silu(qq[i]);
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
        const int c = c0 + u * COLS + cl;
        if (c >= vdim) continue;                            // (sixteen neighbouring lanes together)
        const float v = silu(vv[u]);
        float reads[2] = {0.f, 0.f};
#pragma unroll
        for (int i = 0; i < R; ++i) {
            m[u][i] = fmaf(kk[i], v, decay * m[u][i]);
            reads[i & 1] = fmaf(m[u][i], qq[i], reads[i & 1]);
        }
        float* dst = M + static_cast<size_t>(c) * dim + l * R;
        if constexpr (VEC) {
#pragma unroll
            for (int i = 0; i < R; i += 4)
                if (l * R + i < dim) *reinterpret_cast<float4*>(dst + i) = float4{m[u][i], m[u][i + 1], m[u][i + 2], m[u][i + 3]};
        } else {
#pragma unroll
            for (int i = 0; i < R; ++i)
                if (l * R + i < dim) dst[i] = m[u][i];
        }
        const float read = sum_of_lanes<16>(reads[0] + reads[1]);
        if (l == 0) o[(static_cast<size_t>(t) * in.heads + h) * vdim + c] = read;
    }
}

// out[t] = scale * o[t] / sqrt(mean(o[t]^2) + eps) * w * sigmoid(g[t]) over rows of `width` (all heads side by side): one
// workgroup a row. NV > 0: a thread keeps its values in registers, NV groups of four, everything asked for before anything waits.
template <typename TO, int NV>
__global__ __launch_bounds__(256) void joined_norm_gate_kernel(const float* __restrict__ o, const float* __restrict__ w,
                                                               const float* __restrict__ g, int ld_g, TO* __restrict__ out, int ld_out,
                                                               int width, float eps, float scale) {
    __shared__ float scratch[4];
    const int t = blockIdx.x;
    const float* orow = o + static_cast<size_t>(t) * width;
    const float* grow = g + static_cast<size_t>(t) * ld_g;
    TO* dst = out + static_cast<size_t>(t) * ld_out;
    float ss = 0.f;
    if constexpr (NV > 0) {
        float4 ov[NV], wv[NV], gv[NV];
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const int i = (threadIdx.x + 256 * k) * 4;
            ov[k] = wv[k] = gv[k] = float4{0.f, 0.f, 0.f, 0.f};
            if (i < width) {
                ov[k] = *reinterpret_cast<const float4*>(orow + i);
                wv[k] = *reinterpret_cast<const float4*>(w + i);
                gv[k] = *reinterpret_cast<const float4*>(grow + i);
            }
            ss = fmaf(ov[k].x, ov[k].x, fmaf(ov[k].y, ov[k].y, fmaf(ov[k].z, ov[k].z, fmaf(ov[k].w, ov[k].w, ss))));
        }
        const float inv = scale / sqrtf(block_sum(ss, scratch, 4) / static_cast<float>(width) + eps);
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const int i = (threadIdx.x + 256 * k) * 4;
            if (i >= width) continue;
            struct alignas(sizeof(TO) * 4) Piece { TO x[4]; } y;
            y.x[0] = from_float<TO>((ov[k].x * inv) * wv[k].x / (1.0f + expf(-gv[k].x)));
            y.x[1] = from_float<TO>((ov[k].y * inv) * wv[k].y / (1.0f + expf(-gv[k].y)));
            y.x[2] = from_float<TO>((ov[k].z * inv) * wv[k].z / (1.0f + expf(-gv[k].z)));
            y.x[3] = from_float<TO>((ov[k].w * inv) * wv[k].w / (1.0f + expf(-gv[k].w)));
            *reinterpret_cast<Piece*>(dst + i) = y;
        }
    } else {
        for (int i = threadIdx.x; i < width; i += 256) ss = fmaf(orow[i], orow[i], ss);
        const float inv = scale / sqrtf(block_sum(ss, scratch, 4) / static_cast<float>(width) + eps);
        for (int i = threadIdx.x; i < width; i += 256) dst[i] = from_float<TO>((orow[i] * inv) * w[i] / (1.0f + expf(-grow[i])));
    }
}

// ---------------------------------------------------------------------------------------------------------------
// The chunked form. Chunks of kChunk rows of a request; chunk c of request s has place q_start[s] / kChunk + s + c, which
// no other chunk has.
constexpr int kChunk = 128;

struct LightningChunks {
    float* add;                 // [places, heads, vdim, dim]: what a chunk adds
    bf16* s_hi;                 // [places, heads, vdim, dim]: the memory in front of a chunk, its two parts
    bf16* s_lo;
    int chunk_from;             // requests that bring fewer rows are not taken
};

__device__ __forceinline__ int chunk_place(const int* q_start, int s, int c) { return q_start[s] / kChunk + s + c; }

// a^i for i = 0 .. kChunk into LDS (a^0 is 1 whatever a). No barrier.
__device__ __forceinline__ void decay_powers(const LightningInput& in, int h, float* pw, int tid, int threads) {
    const float log_a = in.decay[in.heads + h];
    for (int i = tid; i <= kChunk; i += threads) pw[i] = i == 0 ? 1.0f : expf(static_cast<float>(i) * log_a);
}

__device__ __forceinline__ void two_parts(float x, bf16& hi, bf16& lo) {
    hi = static_cast<bf16>(x);
    lo = static_cast<bf16>(x - static_cast<float>(hi));
}

// What a chunk adds. A workgroup makes 64 CPW columns (c) of one head's chunk over all key channels (d): wavefront w the
// column tiles w CPW ... Rows (s) come in slabs of 32, turned round as they are staged: K^T [d][s] in one part, the values
// times their power of the decay V^T [c][s] in two. A thread stages pieces of 4 rows x 4 entries; pieces of the same entries
// lie in neighbouring lanes, which keeps the LDS writes free of conflicts.
template <int DT, int CPW>
__global__ __launch_bounds__(256) void lightning_chunk_add_kernel(LightningInput in, const int* __restrict__ q_start, int n_chunks,
                                                                  LightningChunks ck) {
    constexpr int SB = 32, ST = SB + 8;
    constexpr int KP = (DT * 4 * 8 + 255) / 256;            // pieces of keys and of values a thread stages
    constexpr int VP = (64 * CPW / 4 * 8 + 255) / 256;
    __shared__ __align__(16) bf16 k_t[DT * 16 * ST];
    __shared__ __align__(16) bf16 v_hi[64 * CPW * ST];
    __shared__ __align__(16) bf16 v_lo[64 * CPW * ST];
    __shared__ float pw[kChunk + 1];
    const int s = blockIdx.x / n_chunks, c = blockIdx.x % n_chunks, h = blockIdx.y, c0 = blockIdx.z * 64 * CPW;
    const int t0 = q_start[s] + c * kChunk;
    const int n = min(kChunk, q_start[s + 1] - t0);
    if (n <= 0 || q_start[s + 1] - q_start[s] < ck.chunk_from) return;
    const int place = chunk_place(q_start, s, c);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, qd = lane >> 4;
    const int dim = in.dim, vdim = in.vdim;
    decay_powers(in, h, pw, tid, 256);

    const float* kp = in.p + static_cast<size_t>(t0) * in.ld + in.k_col + h * dim;
    const float* vp = in.p + static_cast<size_t>(t0) * in.ld + in.v_col + h * vdim + c0;
    const int vcols = min(64 * CPW, vdim - c0);
    float4 kr[KP][4], vr[VP][4];
    auto fetch = [&](int s0) {
#pragma unroll
        for (int i = 0; i < KP; ++i) {
            const int item = tid + 256 * i, sg = item & 7, d = (item >> 3) * 4;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int row = s0 + sg * 4 + j;
                kr[i][j] = (d < dim && row < n) ? *reinterpret_cast<const float4*>(kp + static_cast<size_t>(row) * in.ld + d)
                                                : float4{0.f, 0.f, 0.f, 0.f};
            }
        }
#pragma unroll
        for (int i = 0; i < VP; ++i) {
            const int item = tid + 256 * i, sg = item & 7, e = (item >> 3) * 4;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int row = s0 + sg * 4 + j;
                vr[i][j] = (e < vcols && row < n) ? *reinterpret_cast<const float4*>(vp + static_cast<size_t>(row) * in.ld + e)
                                                  : float4{0.f, 0.f, 0.f, 0.f};
            }
        }
    };
    auto stage = [&](int s0) {
#pragma unroll
        for (int i = 0; i < KP; ++i) {
            const int item = tid + 256 * i, sg = item & 7, d = (item >> 3) * 4;
            if (d >= DT * 16) continue;
            bf16x4 x[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const float4 k4 = silu4(kr[i][j]);
                x[0][j] = static_cast<bf16>(k4.x);
                x[1][j] = static_cast<bf16>(k4.y);
                x[2][j] = static_cast<bf16>(k4.z);
                x[3][j] = static_cast<bf16>(k4.w);
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) *reinterpret_cast<bf16x4*>(k_t + (d + e) * ST + sg * 4) = x[e];
        }
#pragma unroll
        for (int i = 0; i < VP; ++i) {
            const int item = tid + 256 * i, sg = item & 7, e0 = (item >> 3) * 4;
            if (e0 >= 64 * CPW) continue;
            bf16x4 hi[4], lo[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int row = s0 + sg * 4 + j;
                const float wgt = row < n ? pw[n - 1 - row] : 0.f;
                // (a value enters as bfloat16, then takes its power of the decay)
                const float4 v4 = silu4(vr[i][j]);
                const float x[4] = {v4.x, v4.y, v4.z, v4.w};
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    bf16 a, b;
                    two_parts(static_cast<float>(static_cast<bf16>(x[e])) * wgt, a, b);
                    hi[e][j] = a;
                    lo[e][j] = b;
                }
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                *reinterpret_cast<bf16x4*>(v_hi + (e0 + e) * ST + sg * 4) = hi[e];
                *reinterpret_cast<bf16x4*>(v_lo + (e0 + e) * ST + sg * 4) = lo[e];
            }
        }
    };
    f32x4 acc[CPW][DT];
#pragma unroll
    for (int i = 0; i < CPW; ++i)
#pragma unroll
        for (int j = 0; j < DT; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    fetch(0);
    __syncthreads();                                        // (the powers)
    for (int s0 = 0; s0 < n; s0 += SB) {
        stage(s0);
        __syncthreads();
        if (s0 + SB < n) fetch(s0 + SB);
        bf16x8 fh[CPW], fl[CPW];
#pragma unroll
        for (int i = 0; i < CPW; ++i) {
            fh[i] = *reinterpret_cast<const bf16x8*>(v_hi + ((wave * CPW + i) * 16 + r) * ST + qd * 8);
            fl[i] = *reinterpret_cast<const bf16x8*>(v_lo + ((wave * CPW + i) * 16 + r) * ST + qd * 8);
        }
#pragma unroll
        for (int j = 0; j < DT; ++j) {
            const bf16x8 fk = *reinterpret_cast<const bf16x8*>(k_t + (j * 16 + r) * ST + qd * 8);
#pragma unroll
            for (int i = 0; i < CPW; ++i) {
                acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fh[i], fk, acc[i][j], 0, 0, 0);
                acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fl[i], fk, acc[i][j], 0, 0, 0);
            }
        }
        __syncthreads();
    }
    // acc[i][j]: column (wave CPW + i) 16 + 4 qd + e of the slice, key channel 16 j + r
    float* add = ck.add + (static_cast<size_t>(place) * in.heads + h) * vdim * dim;
#pragma unroll
    for (int i = 0; i < CPW; ++i) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int col = c0 + (wave * CPW + i) * 16 + qd * 4 + e;
            if (col >= vdim) continue;
#pragma unroll
            for (int j = 0; j < DT; ++j)
                if (j * 16 + r < dim) add[static_cast<size_t>(col) * dim + j * 16 + r] = acc[i][j][e];
        }
    }
}

// The memory in front of every chunk and behind the last: one thread per (request, head, column, four key channels).
__global__ __launch_bounds__(256) void lightning_chunk_carry_kernel(float* __restrict__ memory, const float* __restrict__ decay,
                                                                    const int* __restrict__ q_start, const int* __restrict__ slots, int heads,
                                                                    int dim, int vdim, LightningChunks ck) {
    const int s = blockIdx.y;
    const int per_head = vdim * dim;
    const int e = (blockIdx.x * 256 + threadIdx.x) * 4;     // four entries of the request's memory
    if (e >= heads * per_head) return;
    const int h = e / per_head;
    const int rows = q_start[s + 1] - q_start[s];
    const int nc = (rows + kChunk - 1) / kChunk;
    if (nc <= 0 || rows < ck.chunk_from) return;
    const float log_a = decay[heads + h];
    const float whole = expf(static_cast<float>(kChunk) * log_a), rest = expf(static_cast<float>(rows - (nc - 1) * kChunk) * log_a);
    const size_t per = static_cast<size_t>(heads) * per_head;
    float4* slot = reinterpret_cast<float4*>(memory + static_cast<size_t>(slots[s]) * per + e);
    float4 S = *slot;
    const size_t at = static_cast<size_t>(chunk_place(q_start, s, 0)) * per + e;
    constexpr int AHEAD = 8;
    for (int c0 = 0; c0 < nc; c0 += AHEAD) {
        float4 add[AHEAD];
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) {
            if (c0 + i >= nc) break;
            add[i] = *reinterpret_cast<const float4*>(ck.add + at + static_cast<size_t>(c0 + i) * per);
        }
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) {
            if (c0 + i >= nc) break;
            const size_t z = at + static_cast<size_t>(c0 + i) * per;
            const float v[4] = {S.x, S.y, S.z, S.w};
            bf16x4 hi, lo;
#pragma unroll
            for (int x = 0; x < 4; ++x) {
                bf16 a, b;
                two_parts(v[x], a, b);
                hi[x] = a;
                lo[x] = b;
            }
            *reinterpret_cast<bf16x4*>(ck.s_hi + z) = hi;
            *reinterpret_cast<bf16x4*>(ck.s_lo + z) = lo;
            const float keep = c0 + i + 1 < nc ? whole : rest;
            S.x = fmaf(keep, S.x, add[i].x);
            S.y = fmaf(keep, S.y, add[i].y);
            S.z = fmaf(keep, S.z, add[i].z);
            S.w = fmaf(keep, S.w, add[i].w);
        }
    }
    *slot = S;
}

// The rows of half a chunk (64) of one head: NW wavefronts, wavefront w the value tiles w, w + NW, .. (NCT of them) over
// all 64 rows, so that the memory and the values are each read once. The first operand's rows are what is made (values,
// keys), the second operand's columns are the rows t; a lane ends up with row t = 16 rt + r. LDS: Q and K [64][DP + 8],
// V^T [16 tiles][64 + 8], the weights in two parts [64][64 + 8]. DS: slabs of 32 key channels. Everything the first products
// need is asked for before anything waits.
template <int NW, int NCT, int DS>
__global__ __launch_bounds__(NW * 64) void lightning_chunk_read_kernel(LightningInput in, const int* __restrict__ q_start, int n_chunks,
                                                                       LightningChunks ck, float* __restrict__ o) {
    constexpr int NT = NW * 64, KB = 64, KS = KB + 8;
    extern __shared__ __align__(16) unsigned char lds_raw[];
    __shared__ float pw[kChunk + 1];
    const int half = blockIdx.x & 1, sc = blockIdx.x >> 1;
    const int s = sc / n_chunks, c = sc % n_chunks, h = blockIdx.y;
    const int t_chunk = q_start[s] + c * kChunk;
    const int n_chunk = min(kChunk, q_start[s + 1] - t_chunk);      // the chunk's rows
    const int row0 = half * 64;
    if (row0 >= n_chunk || q_start[s + 1] - q_start[s] < ck.chunk_from) return;
    const int n = min(64, n_chunk - row0);                          // this workgroup's rows
    const size_t z = static_cast<size_t>(chunk_place(q_start, s, c)) * in.heads + h;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, qd = lane >> 4;
    const int dim = in.dim, vdim = in.vdim;
    constexpr int DP = DS * 32, QS = DP + 8;
    const int nvt = vdim >> 4;
    bf16* q_l = reinterpret_cast<bf16*>(lds_raw);
    bf16* k_l = q_l + 64 * QS;
    bf16* v_l = k_l + KB * QS;
    bf16* p_hi = v_l + vdim * KS;
    bf16* p_lo = p_hi + 64 * KS;

    // rows [first, first + 64) of the chunk's q or k: pieces of four entries, zeros behind `count` and behind `dim`
    constexpr int PER = DP / 4, QI = 64 * PER / NT;
    auto load_rows = [&](float4 (&x)[QI], int col, int first, int count) {
#pragma unroll
        for (int i = 0; i < QI; ++i) {
            const int item = tid + NT * i, row = item / PER, d = (item % PER) * 4;
            x[i] = (row < count && d < dim)
                       ? *reinterpret_cast<const float4*>(in.p + static_cast<size_t>(t_chunk + first + row) * in.ld + col + h * dim + d)
                       : float4{0.f, 0.f, 0.f, 0.f};
        }
    };
    auto put_rows = [&](bf16* dst, const float4 (&x)[QI]) {
#pragma unroll
        for (int i = 0; i < QI; ++i) {
            const int item = tid + NT * i, row = item / PER, d = (item % PER) * 4;
            const float4 a = silu4(x[i]);
            bf16x4 y;
            y[0] = static_cast<bf16>(a.x);
            y[1] = static_cast<bf16>(a.y);
            y[2] = static_cast<bf16>(a.z);
            y[3] = static_cast<bf16>(a.w);
            *reinterpret_cast<bf16x4*>(dst + row * QS + d) = y;
        }
    };
    // values of rows [first, first + 64), pieces of four rows by four entries, turned round as they are stored
    constexpr int VI = NCT;
    auto load_values = [&](float4 (&x)[VI][4], int first, int count) {
#pragma unroll
        for (int i = 0; i < VI; ++i) {
            const int item = tid + NT * i, sg = item & 15, e0 = (item >> 4) * 4;
#pragma unroll
            for (int j = 0; j < 4; ++j)
                x[i][j] = (e0 < vdim && sg * 4 + j < count)
                              ? *reinterpret_cast<const float4*>(in.p + static_cast<size_t>(t_chunk + first + sg * 4 + j) * in.ld + in.v_col + h * vdim + e0)
                              : float4{0.f, 0.f, 0.f, 0.f};
        }
    };
    auto put_values = [&](const float4 (&v)[VI][4]) {
#pragma unroll
        for (int i = 0; i < VI; ++i) {
            const int item = tid + NT * i, sg = item & 15, e0 = (item >> 4) * 4;
            if (e0 >= vdim) continue;
            bf16x4 x[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const float4 a = silu4(v[i][j]);
                x[0][j] = static_cast<bf16>(a.x);
                x[1][j] = static_cast<bf16>(a.y);
                x[2][j] = static_cast<bf16>(a.z);
                x[3][j] = static_cast<bf16>(a.w);
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) *reinterpret_cast<bf16x4*>(v_l + (e0 + e) * KS + sg * 4) = x[e];
        }
    };
    bf16x8 s_hi[NCT][DS], s_lo[NCT][DS];                    // the memory in front of the chunk, this wavefront's columns
    {
        float4 xq[QI], xk[QI], xv[VI][4];
        load_rows(xq, in.q_col, row0, n);
        load_rows(xk, in.k_col, 0, min(KB, n_chunk));
        load_values(xv, 0, min(KB, n_chunk));
#pragma unroll
        for (int j = 0; j < NCT; ++j) {
            const int ct = wave + NW * j;
#pragma unroll
            for (int k = 0; k < DS; ++k) {
                const int d0 = k * 32 + qd * 8;
#pragma unroll
                for (int e = 0; e < 8; ++e) s_hi[j][k][e] = s_lo[j][k][e] = static_cast<bf16>(0.f);
                if (ct < nvt && d0 < dim) {
                    s_hi[j][k] = *reinterpret_cast<const bf16x8*>(ck.s_hi + (z * vdim + ct * 16 + r) * dim + d0);
                    s_lo[j][k] = *reinterpret_cast<const bf16x8*>(ck.s_lo + (z * vdim + ct * 16 + r) * dim + d0);
                }
            }
        }
        decay_powers(in, h, pw, tid, NT);
        put_rows(q_l, xq);
        put_rows(k_l, xk);
        put_values(xv);
    }
    __syncthreads();

    // the memory in front of the chunk: acc[j][rt] = S_start^T q, times a^(t + 1)
    f32x4 acc[NCT][4];
#pragma unroll
    for (int j = 0; j < NCT; ++j)
#pragma unroll
        for (int rt = 0; rt < 4; ++rt) acc[j][rt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < DS; ++k) {
        bf16x8 fq[4];
#pragma unroll
        for (int rt = 0; rt < 4; ++rt) fq[rt] = *reinterpret_cast<const bf16x8*>(q_l + (rt * 16 + r) * QS + k * 32 + qd * 8);
#pragma unroll
        for (int j = 0; j < NCT; ++j)
#pragma unroll
            for (int rt = 0; rt < 4; ++rt) {
                acc[j][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(s_hi[j][k], fq[rt], acc[j][rt], 0, 0, 0);
                acc[j][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(s_lo[j][k], fq[rt], acc[j][rt], 0, 0, 0);
            }
    }
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) {
        const float w = pw[row0 + rt * 16 + r + 1];
#pragma unroll
        for (int j = 0; j < NCT; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[j][rt][e] *= w;
    }
    // the chunk's own keys, 64 at a time: scores, weights in two parts, their products with the values
    constexpr int KT = 16 / NW;                                             // key tiles of 16 a wavefront scores (of one row tile)
    const int rt_mine = wave & 3, kt0 = (wave >> 2) * KT;
    const int t_mine = row0 + rt_mine * 16 + r;
    for (int key0 = 0; key0 <= row0; key0 += KB) {
        // (the first keys are staged already; the next ones travel while these are worked through)
        const bool more = key0 + KB <= row0;
        float4 xk[QI], xv[VI][4];
        if (more) {
            load_rows(xk, in.k_col, key0 + KB, min(KB, n_chunk - key0 - KB));
            load_values(xv, key0 + KB, min(KB, n_chunk - key0 - KB));
        }
#pragma unroll
        for (int kt = 0; kt < KT; ++kt) {
            f32x4 sc{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < DS; ++k) {
                const int d0 = k * 32 + qd * 8;
                const bf16x8 fk = *reinterpret_cast<const bf16x8*>(k_l + ((kt0 + kt) * 16 + r) * QS + d0);
                const bf16x8 fq = *reinterpret_cast<const bf16x8*>(q_l + (rt_mine * 16 + r) * QS + d0);
                sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fk, fq, sc, 0, 0, 0);
            }
            bf16x4 hi, lo;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int back = t_mine - (key0 + (kt0 + kt) * 16 + qd * 4 + e);
                bf16 a, b;
                two_parts(back >= 0 ? sc[e] * pw[back] : 0.f, a, b);
                hi[e] = a;
                lo[e] = b;
            }
            const int at = (rt_mine * 16 + r) * KS + (kt0 + kt) * 16 + qd * 4;
            *reinterpret_cast<bf16x4*>(p_hi + at) = hi;
            *reinterpret_cast<bf16x4*>(p_lo + at) = lo;
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < KB / 32; ++k) {
            const int s0 = k * 32 + qd * 8;
            bf16x8 fh[4], fl[4];
#pragma unroll
            for (int rt = 0; rt < 4; ++rt) {
                fh[rt] = *reinterpret_cast<const bf16x8*>(p_hi + (rt * 16 + r) * KS + s0);
                fl[rt] = *reinterpret_cast<const bf16x8*>(p_lo + (rt * 16 + r) * KS + s0);
            }
#pragma unroll
            for (int j = 0; j < NCT; ++j) {
                const int ct = wave + NW * j;
                if (ct >= nvt) continue;
                const bf16x8 fv = *reinterpret_cast<const bf16x8*>(v_l + (ct * 16 + r) * KS + s0);
#pragma unroll
                for (int rt = 0; rt < 4; ++rt) {
                    acc[j][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fv, fh[rt], acc[j][rt], 0, 0, 0);
                    acc[j][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fv, fl[rt], acc[j][rt], 0, 0, 0);
                }
            }
        }
        if (more) {
            __syncthreads();                                // (before the next keys take this block's place)
            put_rows(k_l, xk);
            put_values(xv);
            __syncthreads();
        }
    }
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) {
        const int row = rt * 16 + r;
        if (row >= n) continue;
        float* orow = o + (static_cast<size_t>(t_chunk + row0 + row) * in.heads + h) * vdim;
#pragma unroll
        for (int j = 0; j < NCT; ++j) {
            const int ct = wave + NW * j;
            if (ct < nvt) *reinterpret_cast<f32x4*>(orow + ct * 16 + qd * 4) = acc[j][rt];
        }
    }
}

}  // namespace llme

using namespace llme;

// p [T, ld] 32-bit with q, k (heads x dim) and v (heads x vdim), in front of their SiLU, at their columns; decay [2 heads]: the
// decays, then their logarithms; memory [slots, heads, vdim, dim]; o [T, heads vdim] 32-bit. Requests that bring chunk_from
// rows or more are left out (the chunked form takes those and no others).
extern "C" int llme_lightning_walk(const float* p, int ld, int q_col, int k_col, int v_col, const float* decay, int heads, int dim, int vdim,
                                   float* memory, const int* q_start, const int* slots, float* o, int n_seq, int chunk_from,
                                   hipStream_t stream) {
    if (n_seq <= 0) return 0;
    if (heads <= 0 || dim <= 0 || vdim <= 0) return kErrBadArgument;
    if (dim > 256) return kErrUnsupported;
    const LightningInput in{p, ld, q_col, k_col, v_col, decay, heads, dim, vdim};
#define LLME_WALK(R, LPC)                                                                                                                    \
    hipLaunchKernelGGL((lightning_walk_kernel<R, LPC>), dim3((vdim + 256 / LPC - 1) / (256 / LPC), heads, n_seq), dim3(256), 0, stream, in, \
                       memory, q_start, slots, o, chunk_from)
    if (dim <= 16) LLME_WALK(2, 8);
    else if (dim <= 32) LLME_WALK(4, 8);
    else if (dim <= 64) LLME_WALK(4, 16);
    else if (dim <= 128) LLME_WALK(8, 16);
    else LLME_WALK(16, 16);
#undef LLME_WALK
    return launch_status();
}

// A step of one row a request (row s is request s).
extern "C" int llme_lightning_single(const float* p, int ld, int q_col, int k_col, int v_col, const float* decay, int heads, int dim, int vdim,
                                     float* memory, const int* slots, float* o, int T, hipStream_t stream) {
    if (T <= 0) return 0;
    if (heads <= 0 || dim <= 0 || vdim <= 0) return kErrBadArgument;
    if (dim > 256) return kErrUnsupported;
    const LightningInput in{p, ld, q_col, k_col, v_col, decay, heads, dim, vdim};
    const bool vec = dim % 4 == 0 && ld % 4 == 0 && q_col % 4 == 0 && k_col % 4 == 0 && reinterpret_cast<uintptr_t>(p) % 16 == 0 &&
                     reinterpret_cast<uintptr_t>(memory) % 16 == 0;
    const dim3 grid(T, heads, (vdim + 63) / 64);
#define LLME_SINGLE(R)                                                                                                                       \
    do {                                                                                                                                     \
        if (vec) hipLaunchKernelGGL((lightning_single_kernel<R, true>), grid, dim3(256), 0, stream, in, memory, slots, o);                   \
        else hipLaunchKernelGGL((lightning_single_kernel<R, false>), grid, dim3(256), 0, stream, in, memory, slots, o);                      \
    } while (0)
    if (dim <= 64) LLME_SINGLE(4);
    else if (dim <= 128) LLME_SINGLE(8);
    else LLME_SINGLE(16);
#undef LLME_SINGLE
    return launch_status();
}

extern "C" int llme_joined_norm_gate(const float* o, const float* w, const float* g, int ld_g, void* out, int out_dtype, int ld_out, int T,
                                     int width, float eps, float scale, hipStream_t stream) {
    if (T <= 0) return 0;
    if (width <= 0 || ld_g < width || ld_out < width) return kErrBadArgument;
    const bool vec = width % 4 == 0 && width <= 8192 && ld_g % 4 == 0 && ld_out % 4 == 0 && reinterpret_cast<uintptr_t>(o) % 16 == 0 &&
                     reinterpret_cast<uintptr_t>(w) % 16 == 0 && reinterpret_cast<uintptr_t>(g) % 16 == 0 && reinterpret_cast<uintptr_t>(out) % 16 == 0;
    const int nv = !vec ? 0 : width <= 2048 ? 2 : width <= 4096 ? 4 : 8;
#define LLME_JNG(TO, NV)                                                                                                              \
    hipLaunchKernelGGL((joined_norm_gate_kernel<TO, NV>), dim3(T), dim3(256), 0, stream, o, w, g, ld_g, static_cast<TO*>(out), ld_out, \
                       width, eps, scale)
#define LLME_JNG_T(TO)                    \
    do {                                  \
        if (nv == 2) LLME_JNG(TO, 2);     \
        else if (nv == 4) LLME_JNG(TO, 4); \
        else if (nv == 8) LLME_JNG(TO, 8); \
        else LLME_JNG(TO, 0);             \
    } while (0)
    if (out_dtype == kF32) LLME_JNG_T(float);
    else if (out_dtype == kBF16) LLME_JNG_T(bf16);
    else return kErrBadArgument;
#undef LLME_JNG_T
#undef LLME_JNG
    return launch_status();
}

extern "C" int llme_lightning_chunk(void) { return kChunk; }

// The chunked form: p as above with its rows and columns aligned to 16 bytes, dim a multiple of 8 and vdim of 16, both up to
// 256. n_chunks: the most chunks of kChunk rows a request has. add [places, heads, vdim, dim] 32-bit, s_hi and s_lo the same in
// bfloat16: scratch, with places >= T / kChunk + n_seq.
extern "C" int llme_lightning_chunked(const float* p, int ld, int q_col, int k_col, int v_col, const float* decay, int heads, int dim, int vdim,
                                      float* memory, const int* q_start, const int* slots, int n_seq, int n_chunks, int chunk_from, float* add,
                                      void* s_hi, void* s_lo, float* o, hipStream_t stream) {
    if (n_seq <= 0 || n_chunks <= 0) return 0;
    if (heads <= 0 || dim <= 0 || vdim <= 0) return kErrBadArgument;
    if (dim % 8 != 0 || vdim % 16 != 0 || dim > 256 || vdim > 256) return kErrUnsupported;
    if (ld % 4 != 0 || q_col % 4 != 0 || k_col % 4 != 0 || v_col % 4 != 0 || reinterpret_cast<uintptr_t>(p) % 16 != 0) return kErrUnsupported;
    const LightningInput in{p, ld, q_col, k_col, v_col, decay, heads, dim, vdim};
    const LightningChunks ck{add, static_cast<bf16*>(s_hi), static_cast<bf16*>(s_lo), chunk_from};
    const int cpw = vdim >= 128 ? 2 : 1;
    const dim3 add_grid(n_seq * n_chunks, heads, (vdim + 64 * cpw - 1) / (64 * cpw));
#define LLME_ADD(DT)                                                                                                                    \
    do {                                                                                                                                \
        if (cpw == 2) hipLaunchKernelGGL((lightning_chunk_add_kernel<DT, 2>), add_grid, dim3(256), 0, stream, in, q_start, n_chunks, ck); \
        else hipLaunchKernelGGL((lightning_chunk_add_kernel<DT, 1>), add_grid, dim3(256), 0, stream, in, q_start, n_chunks, ck);         \
    } while (0)
    if (dim <= 64) LLME_ADD(4);
    else if (dim <= 128) LLME_ADD(8);
    else LLME_ADD(16);
#undef LLME_ADD
    const int items = heads * vdim * dim / 4;
    hipLaunchKernelGGL(lightning_chunk_carry_kernel, dim3((items + 255) / 256, n_seq), dim3(256), 0, stream, memory, decay, q_start, slots, heads,
                       dim, vdim, ck);
    const int DP = dim <= 64 ? 64 : dim <= 128 ? 128 : 256;
    const int lds = 2 * (2 * 64 * (DP + 8) + vdim * 72 + 2 * 64 * 72);
    const dim3 read_grid(n_seq * n_chunks * 2, heads);
#define LLME_READ_DS(NW, NCT, DS)                                                                                                       \
    do {                                                                                                                                \
        static bool attr_set = false;                                                                                                   \
        if (!attr_set) {                                                                                                                \
            const hipError_t err = hipFuncSetAttribute(reinterpret_cast<const void*>(&lightning_chunk_read_kernel<NW, NCT, DS>),        \
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024);                         \
            if (err != hipSuccess) return static_cast<int>(err);                                                                        \
            attr_set = true;                                                                                                            \
        }                                                                                                                               \
        hipLaunchKernelGGL((lightning_chunk_read_kernel<NW, NCT, DS>), read_grid, dim3(NW * 64), lds, stream, in, q_start, n_chunks, ck, o); \
    } while (0)
#define LLME_READ(NW, NCT)                             \
    do {                                               \
        if (dim <= 64) LLME_READ_DS(NW, NCT, 2);       \
        else if (dim <= 128) LLME_READ_DS(NW, NCT, 4); \
        else LLME_READ_DS(NW, NCT, 8);                 \
    } while (0)
    if (vdim <= 64) LLME_READ(4, 1);
    else if (vdim <= 128) LLME_READ(8, 1);
    else LLME_READ(8, 2);
#undef LLME_READ
#undef LLME_READ_DS
    return launch_status();
}

LLME_LOAD_ENTRY(lightning)
