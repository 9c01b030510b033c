// Matrix memory with exponential gates (the mLSTM of xLSTM). Per request and head a memory S [dim, vdim], a key sum
// z [dim] and a level m, all 32-bit, zero at admission. A token with query q, key k, value v and the logarithms i, f of
// its input and forget gate does
//   m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T;  z <- e^(f + m - m') z + e^(i - m') k;  m <- m'
//   o = S^T (s q) / (max(|z . (s q)|, e^(-m)) + 1e-6)                              (s: a scale on the queries)
// with i = c tanh((a_i + b_i) / c) and f = logsigmoid(c tanh((a_f + b_f) / c)) from the input product's columns a_i, a_f.
// A head's o is then divided by its root mean square, multiplied by a weight and by sigmoid of a gate.
//
// Kept per slot: memory [heads, vdim + 1, dim] with a column's key channels side by side and z as column vdim (a value
// that is always 1), and level [heads, vdim + 1], a copy of m for every column, so that whoever walks a column needs
// nothing that another workgroup writes.
//
// A step in which every request brings one row has a kernel of its own (memory, division, norm and gate in one workgroup a
// head). Otherwise two ways through a request's rows, chosen by how many it brings (`chunk_from`: that many or more are chunked).
// The walk (any sizes, 32-bit throughout; decoded tokens, short portions, the 32-bit model) takes them one by one, columns
// side by side. The chunked form (bfloat16 model, long portions) uses that the rule is linear in S: with b_t the sum of f up to row t of a chunk, a_t = i_t - b_t and M_t = max(m_start, a_1 .. a_t),
//   m_t = b_t + M_t,   S_t = e^(m_start - M_t) S_start + sum_(s <= t) e^(a_s - M_t) k_s v_s^T,
// no exponent is ever positive, and what a row reads is a product with the memory in front of its chunk and a causal
// product with the chunk's own keys and values: three kernels on the matrix cores (v_mfma_f32_16x16x32_bf16).
//   add  : what every chunk adds to an empty memory, sum_s e^(a_s - max a) k_s v_s^T, its (sum of f, max a);
//   carry: chunk by chunk S_start, z_start, m_start of every chunk (S_start as two bfloat16 parts), the slot's new memory;
//   read : the rows of half a chunk: both products, the division, the norm, the gate, the rows in bfloat16.
// q, k and v enter the products as bfloat16 (they are the outputs of a bfloat16 model's projections); everything that is
// weighted (keys times e^(..), scores times e^(..), the memory) enters as the sum of two bfloat16 parts, sums are 32-bit.
#include "common.h"

namespace llme {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
typedef __attribute__((ext_vector_type(4))) float f32x4;

struct MlstmInput {
    const float* p;             // [T, ld]: the input product's rows
    int ld, q_col, k_col, v_col, i_col, f_col;
    const float* bias;          // [2 heads]: the input gates', then the forget gates'
    float cap, q_scale;
    int heads, dim, vdim;
};

__device__ __forceinline__ float capped_gate(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

// ---------------------------------------------------------------------------------------------------------------
// The walk. LPC lanes share a column (lane l holds the R key channels l R ..), a workgroup owns 256 / LPC columns of one
// head of one request. Rows come through LDS in blocks of eight (k, q, the columns' values, the two log gates, which are
// made as a row is staged), the next block asked for while the current one is worked through.
constexpr int kWalkRows = 8;

template <int R, int LPC>
__global__ __launch_bounds__(256) void mlstm_walk_kernel(MlstmInput in, float* __restrict__ memory, float* __restrict__ level,
                                                         const int* __restrict__ q_start, const int* __restrict__ slots,
                                                         float* __restrict__ o, int chunk_from) {
    constexpr int DP = LPC * R, COLS = 256 / LPC;
    constexpr int W = 2 * DP + COLS + 4;                    // floats of a row in LDS: k, q, v, log gates
    constexpr int BLOCK = kWalkRows * W;
    constexpr int NF = (BLOCK + 255) / 256;
    __shared__ __align__(16) float lds[2 * BLOCK];
    const int s = blockIdx.z, h = blockIdx.y, col0 = blockIdx.x * COLS;
    const int tid = threadIdx.x, cl = tid / LPC, l = tid % LPC;
    const int col = col0 + cl;
    const bool live = col <= in.vdim;
    const int first = q_start[s], last = q_start[s + 1];
    if (first >= last || last - first >= chunk_from) return;        // (the whole workgroup)
    const size_t column = (static_cast<size_t>(slots[s]) * in.heads + h) * (in.vdim + 1) + (live ? col : 0);
    float* M = memory + column * in.dim;
    float m[R];
#pragma unroll
    for (int i = 0; i < R; ++i) m[i] = (live && l * R + i < in.dim) ? M[l * R + i] : 0.f;
    float lev = live ? level[column] : 0.f;

    // where each of a thread's NF values of a block comes from: the same column of p for every block of rows
    enum : int { kZero = -1, kOne = -2 };
    int from[NF], row_of[NF];                               // a column of p, or a constant
#pragma unroll
    for (int i = 0; i < NF; ++i) {
        const int e = tid + 256 * i;
        const int x = e % W;
        row_of[i] = e / W;
        from[i] = kZero;
        if (e < BLOCK) {
            if (x < DP) {
                if (x < in.dim) from[i] = in.k_col + h * in.dim + x;
            } else if (x < 2 * DP) {
                if (x - DP < in.dim) from[i] = in.q_col + h * in.dim + x - DP;
            } else if (x < 2 * DP + COLS) {
                const int c = col0 + x - 2 * DP;
                from[i] = c < in.vdim ? in.v_col + h * in.vdim + c : c == in.vdim ? kOne : kZero;
            } else if (x == 2 * DP + COLS) {
                from[i] = in.i_col + h;
            } else if (x == 2 * DP + COLS + 1) {
                from[i] = in.f_col + h;
            }
        }
    }
    const float bias_i = in.bias[h], bias_f = in.bias[in.heads + h];
    float pre[NF];
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < NF; ++i) {
            const int t = t0 + row_of[i];
            pre[i] = from[i] == kOne ? 1.f : (from[i] >= 0 && t < last) ? in.p[static_cast<size_t>(t) * in.ld + from[i]] : 0.f;
        }
    };
    auto put = [&](int buf) {
#pragma unroll
        for (int i = 0; i < NF; ++i) {
            const int e = tid + 256 * i;
            if (e >= BLOCK) continue;
            float v = pre[i];
            if (from[i] == in.i_col + h) v = capped_gate(v + bias_i, in.cap);
            else if (from[i] == in.f_col + h) v = log_sigmoid(capped_gate(v + bias_f, in.cap));
            lds[buf * BLOCK + e] = v;
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
            const float li = row[2 * DP + COLS], lf = row[2 * DP + COLS + 1];
            const float top = fmaxf(lf + lev, li);
            const float keep = expf(lf + lev - top);
            const float w = expf(li - top) * row[2 * DP + cl];
            lev = top;
            float reads[2] = {0.f, 0.f};
#pragma unroll
            for (int i = 0; i < R; i += 2) {
                const float2 k2 = *reinterpret_cast<const float2*>(row + l * R + i);
                const float2 q2 = *reinterpret_cast<const float2*>(row + DP + l * R + i);
                m[i] = fmaf(k2.x, w, keep * m[i]);
                m[i + 1] = fmaf(k2.y, w, keep * m[i + 1]);
                reads[0] = fmaf(m[i], q2.x, reads[0]);
                reads[1] = fmaf(m[i + 1], q2.y, reads[1]);
            }
            const float read = sum_of_lanes<LPC>(reads[0] + reads[1]) * in.q_scale;
            if (live && l == 0) {
                float* orow = o + (static_cast<size_t>(t0 + tt) * in.heads + h) * (in.vdim + 2);
                orow[col] = read;
                if (col == in.vdim) orow[col + 1] = lev;
            }
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
    if (live && l == 0) level[column] = lev;
}

// What the walk left of a row, [T, heads, vdim + 2] (the unscaled reads, z . q, m), to the mixer's row: one wavefront per
// (row, head). out = scale * (o / rms(o)) * w * sigmoid(g), o = reads / (max(|z . q|, e^-m) + 1e-6).
template <typename TO>
__global__ __launch_bounds__(256) void mlstm_finish_kernel(const float* __restrict__ o, const float* __restrict__ w,
                                                           const float* __restrict__ g, int ld_g, TO* __restrict__ out, int ld_out,
                                                           int T, int heads, int vdim, float eps, float scale,
                                                           const int* __restrict__ seq_idx, const int* __restrict__ q_start,
                                                           int chunk_from) {
    const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
    const int item = blockIdx.x * 4 + wave;
    if (item >= T * heads) return;
    const int t = item / heads, h = item % heads;
    if (q_start[seq_idx[t] + 1] - q_start[seq_idx[t]] >= chunk_from) return;
    const float* p = o + static_cast<size_t>(item) * (vdim + 2);
    const float inv_den = 1.0f / (fmaxf(fabsf(p[vdim]), expf(-p[vdim + 1])) + 1e-6f);
    float ss = 0.f;
    for (int j = lane; j < vdim; j += kWave) {
        const float v = p[j] * inv_den;
        ss = fmaf(v, v, ss);
    }
    const float inv = scale * inv_den / sqrtf(wave_sum(ss) / static_cast<float>(vdim) + eps);
    for (int j = lane; j < vdim; j += kWave) {
        const float z = g[static_cast<size_t>(t) * ld_g + h * vdim + j];
        out[static_cast<size_t>(t) * ld_out + h * vdim + j] = from_float<TO>((p[j] * inv) * w[h * vdim + j] / (1.0f + expf(-z)));
    }
}

// A step in which every request brings one row (decoding): one workgroup of 1,024 threads per (request, head) takes the row
// through the whole memory and finishes it, so that nothing is passed on. 16 lanes share a column (R key channels each), 64
// columns a pass, four passes' columns asked for together. VEC: channels come in whole pieces of four.
template <int R, bool VEC, typename TO>
__global__ __launch_bounds__(1024) void mlstm_single_kernel(MlstmInput in, float* __restrict__ memory, float* __restrict__ level,
                                                            const int* __restrict__ slots, const float* __restrict__ norm_w, int g_col,
                                                            float eps, float scale, TO* __restrict__ out, int ld_out) {
    constexpr int COLS = 64, U = R >= 16 ? 2 : 4;
    extern __shared__ float read_s[];                       // [vdim + 1]
    __shared__ float scratch[16];
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    const int cl = tid >> 4, l = tid & 15, vdim = in.vdim, dim = in.dim;
    const float* row = in.p + static_cast<size_t>(t) * in.ld;
    const size_t column0 = (static_cast<size_t>(slots[t]) * in.heads + h) * (vdim + 1);
    float kk[R], qq[R];
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
    load(row + in.k_col + h * dim, kk);
    load(row + in.q_col + h * dim, qq);
    const float li = capped_gate(row[in.i_col + h] + in.bias[h], in.cap);
    const float lf = log_sigmoid(capped_gate(row[in.f_col + h] + in.bias[in.heads + h], in.cap));
    const float lev = level[column0];                       // (a copy for every column; this workgroup is the only one that takes them)
    const float top = fmaxf(lf + lev, li);
    const float keep = expf(lf + lev - top), add = expf(li - top);
    for (int c0 = 0; c0 < vdim; c0 += COLS * U) {
        // (place U of the first pass: the key sum, column vdim, by the first sixteen lanes)
        float m[U + 1][R], vv[U + 1];
#pragma unroll
        for (int u = 0; u <= U; ++u) {
            const int c = u < U ? c0 + u * COLS + cl : vdim;
            const bool mine = u < U ? c < vdim : c0 == 0 && cl == 0;
            vv[u] = mine && u < U ? row[in.v_col + h * vdim + c] : 1.f;
            if (mine) load(memory + (column0 + c) * dim, m[u]);
        }
#pragma unroll
        for (int u = 0; u <= U; ++u) {
            const int c = u < U ? c0 + u * COLS + cl : vdim;
            if (!(u < U ? c < vdim : c0 == 0 && cl == 0)) continue;         // (sixteen neighbouring lanes together)
            const float w = add * vv[u];
            float reads[2] = {0.f, 0.f};
#pragma unroll
            for (int i = 0; i < R; ++i) {
                m[u][i] = fmaf(kk[i], w, keep * m[u][i]);
                reads[i & 1] = fmaf(m[u][i], qq[i], reads[i & 1]);
            }
            float* M = memory + (column0 + c) * dim + l * R;
            if constexpr (VEC) {
#pragma unroll
                for (int i = 0; i < R; i += 4)
                    if (l * R + i < dim) *reinterpret_cast<float4*>(M + i) = float4{m[u][i], m[u][i + 1], m[u][i + 2], m[u][i + 3]};
            } else {
#pragma unroll
                for (int i = 0; i < R; ++i)
                    if (l * R + i < dim) M[i] = m[u][i];
            }
            const float read = sum_of_lanes<16>(reads[0] + reads[1]) * in.q_scale;
            if (l == 0) read_s[c] = read;
        }
    }
    __syncthreads();                                        // (every thread has read the level by now)
    for (int c = tid; c <= vdim; c += 1024) level[column0 + c] = top;
    const float inv_den = 1.0f / (fmaxf(fabsf(read_s[vdim]), expf(-top)) + 1e-6f);
    float ss = 0.f;
    for (int c = tid; c < vdim; c += 1024) {
        const float v = read_s[c] * inv_den;
        ss = fmaf(v, v, ss);
    }
    const float inv = scale * inv_den / sqrtf(block_sum(ss, scratch, 16) / static_cast<float>(vdim) + eps);
    for (int c = tid; c < vdim; c += 1024) {
        const float z = row[g_col + h * vdim + c];
        out[static_cast<size_t>(t) * ld_out + h * vdim + c] = from_float<TO>((read_s[c] * inv) * norm_w[h * vdim + c] / (1.0f + expf(-z)));
    }
}

// ---------------------------------------------------------------------------------------------------------------
// The chunked form. Chunks of kChunk rows of a request; chunk c of request s has place q_start[s] / kChunk + s + c, which
// no other chunk has.
constexpr int kChunk = 128;

struct MlstmChunks {
    float* add;                 // [places, heads, vdim + 1, dim]: what a chunk adds (row vdim: to z)
    float* ends;                // [places, heads, 2]: the chunk's sum of f, its largest a
    int chunk_from;             // requests that bring fewer rows are not taken
    bf16* s_hi;                 // [places, heads, vdim, dim]: the memory in front of a chunk, its two parts
    bf16* s_lo;
    float* z;                   // [places, heads, dim]: the key sum in front of a chunk
    float* m;                   // [places, heads]: the level in front of a chunk
};

__device__ __forceinline__ int chunk_place(const int* q_start, int s, int c) { return q_start[s] / kChunk + s + c; }

// b (sums of f from the chunk's start, inclusive) and a = i - b of a chunk's rows into LDS arrays of kChunk; M receives the
// running maximum of a (from -inf). Rows behind the chunk's n have a = -inf. Needs at least kChunk threads; has barriers.
__device__ __forceinline__ void chunk_gates(const MlstmInput& in, int h, int t0, int n, float* b_s, float* a_s, float* M_s,
                                            float* scratch) {
    const int tid = threadIdx.x, lane = tid & 63;
    float li = -INFINITY, b = 0.f;
    if (tid < n) {
        const float* row = in.p + static_cast<size_t>(t0 + tid) * in.ld;
        li = capped_gate(row[in.i_col + h] + in.bias[h], in.cap);
        b = log_sigmoid(capped_gate(row[in.f_col + h] + in.bias[in.heads + h], in.cap));
    }
#pragma unroll
    for (int off = 1; off < kWave; off <<= 1) {
        const float o = __shfl_up(b, off, kWave);
        if (lane >= off) b += o;
    }
    if (tid == kWave - 1) scratch[0] = b;
    __syncthreads();
    if (tid >= kWave && tid < kChunk) b += scratch[0];
    const float a = li - b;
    float mx = a;
#pragma unroll
    for (int off = 1; off < kWave; off <<= 1) {
        const float o = __shfl_up(mx, off, kWave);
        if (lane >= off) mx = fmaxf(mx, o);
    }
    if (tid == kWave - 1) scratch[1] = mx;
    __syncthreads();
    if (tid >= kWave && tid < kChunk) mx = fmaxf(mx, scratch[1]);
    if (tid < kChunk) {
        b_s[tid] = b;
        a_s[tid] = a;
        M_s[tid] = mx;
    }
    __syncthreads();
}

// What a chunk adds. A workgroup makes 64 CPW columns (c) of one head's chunk over all key channels (d): wavefront w the
// column tiles w CPW ... Rows (s) come in slabs of 32, turned round as they are staged: V^T [c][s] in one part, the weighted
// keys K^T [d][s] in two. A thread stages pieces of 4 rows x 4 entries; pieces of the same entries lie in neighbouring lanes,
// which keeps the LDS writes free of conflicts.
template <int DT, int CPW>
__global__ __launch_bounds__(256) void mlstm_chunk_add_kernel(MlstmInput in, const int* __restrict__ q_start, int n_chunks,
                                                              MlstmChunks ck) {
    constexpr int SB = 32, ST = SB + 8;
    constexpr int KP = (DT * 4 * 8 + 255) / 256;            // pieces of keys and of values a thread stages
    constexpr int VP = (64 * CPW / 4 * 8 + 255) / 256;
    __shared__ __align__(16) bf16 k_hi[DT * 16 * ST];
    __shared__ __align__(16) bf16 k_lo[DT * 16 * ST];
    __shared__ __align__(16) bf16 v_t[64 * CPW * ST];
    __shared__ float b_s[kChunk], a_s[kChunk], M_s[kChunk], scratch[2];
    const int s = blockIdx.x / n_chunks, c = blockIdx.x % n_chunks, h = blockIdx.y, c0 = blockIdx.z * 64 * CPW;
    const int t0 = q_start[s] + c * kChunk;
    const int n = min(kChunk, q_start[s + 1] - t0);
    if (n <= 0 || q_start[s + 1] - q_start[s] < ck.chunk_from) return;
    const int place = chunk_place(q_start, s, c);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, qd = lane >> 4;
    const int dim = in.dim, vdim = in.vdim;
    chunk_gates(in, h, t0, n, b_s, a_s, M_s, scratch);
    const float a_max = M_s[n - 1];

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
    float z_acc[KP][4];
#pragma unroll
    for (int i = 0; i < KP; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) z_acc[i][e] = 0.f;
    auto stage = [&](int s0) {
#pragma unroll
        for (int i = 0; i < KP; ++i) {
            const int item = tid + 256 * i, sg = item & 7, d = (item >> 3) * 4;
            if (d >= DT * 16) continue;
            bf16x4 hi[4], lo[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int row = s0 + sg * 4 + j;
                const float wgt = row < n ? expf(a_s[row < kChunk ? row : 0] - a_max) : 0.f;
                const float x[4] = {kr[i][j].x * wgt, kr[i][j].y * wgt, kr[i][j].z * wgt, kr[i][j].w * wgt};
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    z_acc[i][e] += x[e];
                    const bf16 top = static_cast<bf16>(x[e]);
                    hi[e][j] = top;
                    lo[e][j] = static_cast<bf16>(x[e] - static_cast<float>(top));
                }
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                *reinterpret_cast<bf16x4*>(k_hi + (d + e) * ST + sg * 4) = hi[e];
                *reinterpret_cast<bf16x4*>(k_lo + (d + e) * ST + sg * 4) = lo[e];
            }
        }
#pragma unroll
        for (int i = 0; i < VP; ++i) {
            const int item = tid + 256 * i, sg = item & 7, e0 = (item >> 3) * 4;
            if (e0 >= 64 * CPW) continue;
            bf16x4 x[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                x[0][j] = static_cast<bf16>(vr[i][j].x);
                x[1][j] = static_cast<bf16>(vr[i][j].y);
                x[2][j] = static_cast<bf16>(vr[i][j].z);
                x[3][j] = static_cast<bf16>(vr[i][j].w);
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) *reinterpret_cast<bf16x4*>(v_t + (e0 + e) * ST + sg * 4) = x[e];
        }
    };
    f32x4 acc[CPW][DT];
#pragma unroll
    for (int i = 0; i < CPW; ++i)
#pragma unroll
        for (int j = 0; j < DT; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    fetch(0);
    for (int s0 = 0; s0 < n; s0 += SB) {
        stage(s0);
        __syncthreads();
        if (s0 + SB < n) fetch(s0 + SB);
        bf16x8 fv[CPW];
#pragma unroll
        for (int i = 0; i < CPW; ++i) fv[i] = *reinterpret_cast<const bf16x8*>(v_t + ((wave * CPW + i) * 16 + r) * ST + qd * 8);
#pragma unroll
        for (int j = 0; j < DT; ++j) {
            const bf16x8 fh = *reinterpret_cast<const bf16x8*>(k_hi + (j * 16 + r) * ST + qd * 8);
            const bf16x8 fl = *reinterpret_cast<const bf16x8*>(k_lo + (j * 16 + r) * ST + qd * 8);
#pragma unroll
            for (int i = 0; i < CPW; ++i) {
                acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fv[i], fh, acc[i][j], 0, 0, 0);
                acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fv[i], fl, acc[i][j], 0, 0, 0);
            }
        }
        __syncthreads();
    }
    // acc[i][j]: column (wave CPW + i) 16 + 4 qd + e of the slice, key channel 16 j + r
    float* add = ck.add + (static_cast<size_t>(place) * in.heads + h) * (vdim + 1) * dim;
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
    if (blockIdx.z == 0) {
#pragma unroll
        for (int i = 0; i < KP; ++i) {
            const int d = ((tid + 256 * i) >> 3) * 4;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float v = sum_of_lanes<8>(z_acc[i][e]);       // the pieces of the same channels: eight neighbouring lanes
                if ((lane & 7) == 0 && d + e < dim) add[static_cast<size_t>(vdim) * dim + d + e] = v;
            }
        }
        if (tid == 0) {
            ck.ends[(static_cast<size_t>(place) * in.heads + h) * 2] = b_s[n - 1];
            ck.ends[(static_cast<size_t>(place) * in.heads + h) * 2 + 1] = a_max;
        }
    }
}

// The memory in front of every chunk and behind the last: one thread per (request, head, column, four key channels).
__global__ __launch_bounds__(256) void mlstm_chunk_carry_kernel(float* __restrict__ memory, const float* __restrict__ level,
                                                                const int* __restrict__ q_start, const int* __restrict__ slots, int heads,
                                                                int dim, int vdim, MlstmChunks ck) {
    const int s = blockIdx.y;
    const int d4 = dim / 4;
    const int e = blockIdx.x * 256 + threadIdx.x;
    if (e >= heads * (vdim + 1) * d4) return;
    const int d = (e % d4) * 4, col = (e / d4) % (vdim + 1), h = e / d4 / (vdim + 1);
    const int rows = q_start[s + 1] - q_start[s];
    const int nc = (rows + kChunk - 1) / kChunk;
    if (nc <= 0 || rows < ck.chunk_from) return;
    const size_t column = (static_cast<size_t>(slots[s]) * heads + h) * (vdim + 1) + col;
    float4* slot = reinterpret_cast<float4*>(memory + column * dim + d);
    float4 S = *slot;
    float m = level[column];            // (the next kernel writes the new one: other threads still read this one)
    size_t at = static_cast<size_t>(chunk_place(q_start, s, 0)) * heads + h;
    constexpr int AHEAD = 8;
    for (int c0 = 0; c0 < nc; c0 += AHEAD) {
        float4 add[AHEAD];
        float end[AHEAD], top[AHEAD];
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) {
            if (c0 + i >= nc) break;
            const size_t z = at + static_cast<size_t>(c0 + i) * heads;
            add[i] = *reinterpret_cast<const float4*>(ck.add + (z * (vdim + 1) + col) * dim + d);
            end[i] = ck.ends[z * 2];
            top[i] = ck.ends[z * 2 + 1];
        }
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) {
            if (c0 + i >= nc) break;
            const size_t z = at + static_cast<size_t>(c0 + i) * heads;
            const float v[4] = {S.x, S.y, S.z, S.w};
            if (col < vdim) {
                bf16x4 hi, lo;
#pragma unroll
                for (int x = 0; x < 4; ++x) {
                    hi[x] = static_cast<bf16>(v[x]);
                    lo[x] = static_cast<bf16>(v[x] - static_cast<float>(hi[x]));
                }
                *reinterpret_cast<bf16x4*>(ck.s_hi + (z * vdim + col) * dim + d) = hi;
                *reinterpret_cast<bf16x4*>(ck.s_lo + (z * vdim + col) * dim + d) = lo;
            } else {
                *reinterpret_cast<float4*>(ck.z + z * dim + d) = S;
                if (d == 0) ck.m[z] = m;
            }
            const float M = fmaxf(m, top[i]);
            const float keep = expf(m - M), take = expf(top[i] - M);
            S.x = fmaf(take, add[i].x, keep * S.x);
            S.y = fmaf(take, add[i].y, keep * S.y);
            S.z = fmaf(take, add[i].z, keep * S.z);
            S.w = fmaf(take, add[i].w, keep * S.w);
            m = end[i] + M;
        }
    }
    *slot = S;
}

// The rows of half a chunk (64) of one head: NW wavefronts, wavefront w the value tiles w, w + NW, .. (NCT of them) over
// all 64 rows, so that the memory and the values are each read once. Products as in the attention kernels: the first
// operand's rows are what is made (values, keys), the second operand's columns are the rows t; a lane ends up with row
// t = 16 rt + r. LDS: Q and K [64][DP + 8], V^T [16 tiles][64 + 8], the weights in two parts [64][64 + 8]. DS: slabs of 32
// key channels. Everything the first products need is asked for before anything waits; the workgroup of a request's last
// chunk also leaves the slot's new level.
template <int NW, int NCT, int DS>
__global__ __launch_bounds__(NW * 64) void mlstm_chunk_read_kernel(MlstmInput in, const int* __restrict__ q_start, int n_chunks,
                                                                   const int* __restrict__ slots, float* __restrict__ level, MlstmChunks ck, const float* __restrict__ norm_w, int g_col, float eps,
                                                                   float scale, bf16* __restrict__ out, int ld_out) {
    constexpr int NT = NW * 64, KB = 64, KS = KB + 8;
    extern __shared__ __align__(16) unsigned char lds_raw[];
    __shared__ float b_s[kChunk], a_s[kChunk], M_s[kChunk], scratch[2], z_s[256];
    __shared__ float row_sum[2][64], row_z[64], row_ss[NW][64];
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
            bf16x4 y;
            y[0] = static_cast<bf16>(x[i].x);
            y[1] = static_cast<bf16>(x[i].y);
            y[2] = static_cast<bf16>(x[i].z);
            y[3] = static_cast<bf16>(x[i].w);
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
                x[0][j] = static_cast<bf16>(v[i][j].x);
                x[1][j] = static_cast<bf16>(v[i][j].y);
                x[2][j] = static_cast<bf16>(v[i][j].z);
                x[3][j] = static_cast<bf16>(v[i][j].w);
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) *reinterpret_cast<bf16x4*>(v_l + (e0 + e) * KS + sg * 4) = x[e];
        }
    };
    bf16x8 s_hi[NCT][DS], s_lo[NCT][DS];                    // the memory in front of the chunk, this wavefront's columns
    const float m_start = ck.m[z];
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
        put_rows(q_l, xq);
        put_rows(k_l, xk);
        put_values(xv);
    }
    for (int d = tid; d < dim; d += NT) z_s[d] = ck.z[z * dim + d];
    if (half == 0 && t_chunk + n_chunk == q_start[s + 1]) {
        const float m_end = ck.ends[z * 2] + fmaxf(m_start, ck.ends[z * 2 + 1]);
        float* lev = level + (static_cast<size_t>(slots[s]) * in.heads + h) * (vdim + 1);
        for (int col = tid; col <= vdim; col += NT) lev[col] = m_end;
    }
    chunk_gates(in, h, t_chunk, n_chunk, b_s, a_s, M_s, scratch);           // (its barriers also cover the staged rows)

    // the memory in front of the chunk: acc[j][rt] = S_start^T q
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
    float M_row[4], start_w[4];                                             // of this lane's rows
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) {
        M_row[rt] = fmaxf(m_start, M_s[row0 + rt * 16 + r]);
        start_w[rt] = expf(m_start - M_row[rt]) * in.q_scale;
#pragma unroll
        for (int j = 0; j < NCT; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[j][rt][e] *= start_w[rt];
    }
    // z_start . q of every row: four lanes a row
    if (tid < 256) {
        const int row = tid >> 2, part = tid & 3;
        float v = 0.f;
        for (int d = part; d < dim; d += 4) v = fmaf(static_cast<float>(q_l[row * QS + d]), z_s[d], v);
        v += __shfl_xor(v, 1, kWave);
        v += __shfl_xor(v, 2, kWave);
        if (part == 0) row_z[row] = v;
    }
    // the chunk's own keys, 64 at a time: scores, weights in two parts, their products with the values
    constexpr int KT = 16 / NW;                                             // key tiles of 16 a wavefront scores (of one row tile)
    const int rt_mine = wave & 3, kt0 = (wave >> 2) * KT;
    const float M_mine = M_row[rt_mine];
    float sum = 0.f;
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
                const int key = key0 + (kt0 + kt) * 16 + qd * 4 + e;
                const float w = key <= row0 + rt_mine * 16 + r ? sc[e] * in.q_scale * expf(a_s[key] - M_mine) : 0.f;
                sum += w;
                hi[e] = static_cast<bf16>(w);
                lo[e] = static_cast<bf16>(w - static_cast<float>(hi[e]));
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
    sum += __shfl_xor(sum, 16, kWave);
    sum += __shfl_xor(sum, 32, kWave);
    if (qd == 0) row_sum[wave >> 2][rt_mine * 16 + r] = sum;
    __syncthreads();
    // the division, the norm over the head's entries, weight and gate
    float ss[4];
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) {
        const int row = rt * 16 + r;
        const float zq = (NW > 4 ? row_sum[0][row] + row_sum[1][row] : row_sum[0][row]) + start_w[rt] * row_z[row];
        const float m_row = b_s[row0 + row] + M_row[rt];
        const float inv_den = 1.0f / (fmaxf(fabsf(zq), expf(-m_row)) + 1e-6f);
        ss[rt] = 0.f;
#pragma unroll
        for (int j = 0; j < NCT; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                acc[j][rt][e] *= inv_den;
                ss[rt] = fmaf(acc[j][rt][e], acc[j][rt][e], ss[rt]);
            }
        ss[rt] += __shfl_xor(ss[rt], 16, kWave);
        ss[rt] += __shfl_xor(ss[rt], 32, kWave);
        if (qd == 0) row_ss[wave][row] = ss[rt];
    }
    __syncthreads();
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) {
        const int row = rt * 16 + r;
        if (row >= n) continue;
        float total = 0.f;
#pragma unroll
        for (int w = 0; w < NW; ++w) total += row_ss[w][row];
        const float inv = scale / sqrtf(total / static_cast<float>(vdim) + eps);
        const size_t t = static_cast<size_t>(t_chunk + row0 + row);
#pragma unroll
        for (int j = 0; j < NCT; ++j) {
            const int ct = wave + NW * j;
            if (ct >= nvt) continue;
            const int col = h * vdim + ct * 16 + qd * 4;
            const float4 g = *reinterpret_cast<const float4*>(in.p + t * in.ld + g_col + col);
            const float4 w = *reinterpret_cast<const float4*>(norm_w + col);
            const float gv[4] = {g.x, g.y, g.z, g.w}, wv[4] = {w.x, w.y, w.z, w.w};
            bf16x4 y;
#pragma unroll
            for (int e = 0; e < 4; ++e) y[e] = static_cast<bf16>((acc[j][rt][e] * inv) * wv[e] / (1.0f + expf(-gv[e])));
            *reinterpret_cast<bf16x4*>(out + t * ld_out + col) = y;
        }
    }
}

}  // namespace llme

using namespace llme;

static MlstmInput mlstm_input(const float* p, int ld, int q_col, int k_col, int v_col, int i_col, int f_col, const float* bias, float cap,
                              float q_scale, int heads, int dim, int vdim) {
    return MlstmInput{p, ld, q_col, k_col, v_col, i_col, f_col, bias, cap, q_scale, heads, dim, vdim};
}

// p [T, ld] 32-bit with q, k (heads x dim), v (heads x vdim) and the gates' sums (heads each) at their columns; bias
// [2 heads]; memory [slots, heads, vdim + 1, dim], level [slots, heads, vdim + 1]; o [T, heads, vdim + 2] 32-bit. Requests
// that bring chunk_from rows or more are left out (also by llme_mlstm_finish; the chunked form takes those and no others).
extern "C" int llme_mlstm_walk(const float* p, int ld, int q_col, int k_col, int v_col, int i_col, int f_col, const float* bias, float cap,
                               float q_scale, int heads, int dim, int vdim, float* memory, float* level, const int* q_start,
                               const int* slots, float* o, int n_seq, int chunk_from, hipStream_t stream) {
    if (n_seq <= 0) return 0;
    if (heads <= 0 || dim <= 0 || vdim <= 0 || !(cap > 0.f)) return kErrBadArgument;
    if (dim > 256) return kErrUnsupported;
    const MlstmInput in = mlstm_input(p, ld, q_col, k_col, v_col, i_col, f_col, bias, cap, q_scale, heads, dim, vdim);
#define LLME_WALK(R, LPC)                                                                                            \
    hipLaunchKernelGGL((mlstm_walk_kernel<R, LPC>), dim3((vdim + 1 + 256 / LPC - 1) / (256 / LPC), heads, n_seq), dim3(256), 0, stream, \
                       in, memory, level, q_start, slots, o, chunk_from)
    if (dim <= 16) LLME_WALK(2, 8);
    else if (dim <= 32) LLME_WALK(4, 8);
    else if (dim <= 64) LLME_WALK(4, 16);
    else if (dim <= 128) LLME_WALK(8, 16);
    else LLME_WALK(16, 16);
#undef LLME_WALK
    return launch_status();
}

extern "C" int llme_mlstm_finish(const float* o, const float* w, const float* g, int ld_g, void* out, int out_dtype, int ld_out, int T,
                                 int heads, int vdim, float eps, float scale, const int* seq_idx, const int* q_start, int chunk_from,
                                 hipStream_t stream) {
    const long items = static_cast<long>(T) * heads;
    if (items <= 0) return 0;
    if (vdim <= 0) return kErrBadArgument;
    const dim3 grid(static_cast<unsigned>((items + 3) / 4));
    if (out_dtype == kF32)
        hipLaunchKernelGGL((mlstm_finish_kernel<float>), grid, dim3(256), 0, stream, o, w, g, ld_g, static_cast<float*>(out), ld_out, T,
                           heads, vdim, eps, scale, seq_idx, q_start, chunk_from);
    else if (out_dtype == kBF16)
        hipLaunchKernelGGL((mlstm_finish_kernel<bf16>), grid, dim3(256), 0, stream, o, w, g, ld_g, static_cast<bf16*>(out), ld_out, T,
                           heads, vdim, eps, scale, seq_idx, q_start, chunk_from);
    else return kErrBadArgument;
    return launch_status();
}

// A step of one row a request (row s is request s): the row through the memory and finished. out [T, ld_out] in out_dtype, the
// gate's sums at g_col of p.
extern "C" int llme_mlstm_single(const float* p, int ld, int q_col, int k_col, int v_col, int g_col, int i_col, int f_col, const float* bias,
                                 float cap, float q_scale, int heads, int dim, int vdim, float* memory, float* level, const int* slots, int T,
                                 const float* norm_w, float eps, float scale, void* out, int out_dtype, int ld_out, hipStream_t stream) {
    if (T <= 0) return 0;
    if (heads <= 0 || dim <= 0 || vdim <= 0 || !(cap > 0.f)) return kErrBadArgument;
    if (dim > 256 || vdim > 8192) return kErrUnsupported;
    const MlstmInput in = mlstm_input(p, ld, q_col, k_col, v_col, i_col, f_col, bias, cap, q_scale, heads, dim, vdim);
    const bool vec = dim % 4 == 0 && ld % 4 == 0 && q_col % 4 == 0 && k_col % 4 == 0 && reinterpret_cast<uintptr_t>(p) % 16 == 0 &&
                     reinterpret_cast<uintptr_t>(memory) % 16 == 0;
    const size_t lds = static_cast<size_t>(vdim + 1) * 4;
#define LLME_SINGLE_T(R, VEC, TO)                                                                                                    \
    hipLaunchKernelGGL((mlstm_single_kernel<R, VEC, TO>), dim3(T, heads), dim3(1024), lds, stream, in, memory, level, slots, norm_w, \
                       g_col, eps, scale, static_cast<TO*>(out), ld_out)
#define LLME_SINGLE(R)                                                  \
    do {                                                                \
        if (vec && out_dtype == kF32) LLME_SINGLE_T(R, true, float);    \
        else if (vec) LLME_SINGLE_T(R, true, bf16);                     \
        else if (out_dtype == kF32) LLME_SINGLE_T(R, false, float);     \
        else LLME_SINGLE_T(R, false, bf16);                             \
    } while (0)
    if (out_dtype != kF32 && out_dtype != kBF16) return kErrBadArgument;
    if (dim <= 64) LLME_SINGLE(4);
    else if (dim <= 128) LLME_SINGLE(8);
    else LLME_SINGLE(16);
#undef LLME_SINGLE
#undef LLME_SINGLE_T
    return launch_status();
}

extern "C" int llme_mlstm_chunk(void) { return kChunk; }

// The chunked form: p as above with its rows and columns aligned to 16 bytes, dim a multiple of 8 and vdim of 16, both up
// to 256. n_chunks: the most chunks of kChunk rows a request has. add [places, heads, vdim + 1, dim], ends [places, heads, 2],
// s_hi and s_lo [places, heads, vdim, dim] bfloat16, z [places, heads, dim], m [places, heads]: scratch, with
// places >= T / kChunk + n_seq. out [T, ld_out] bfloat16 at 8-byte boundaries; the gate's sums at g_col of p.
extern "C" int llme_mlstm_chunked(const float* p, int ld, int q_col, int k_col, int v_col, int g_col, int i_col, int f_col, const float* bias,
                                  float cap, float q_scale, int heads, int dim, int vdim, float* memory, float* level, const int* q_start,
                                  const int* slots, int n_seq, int n_chunks, int chunk_from, float* add, float* ends, void* s_hi, void* s_lo, float* z,
                                  float* m, const float* norm_w, float eps, float scale, void* out, int ld_out, hipStream_t stream) {
    if (n_seq <= 0 || n_chunks <= 0) return 0;
    if (heads <= 0 || dim <= 0 || vdim <= 0 || !(cap > 0.f)) return kErrBadArgument;
    if (dim % 8 != 0 || vdim % 16 != 0 || dim > 256 || vdim > 256) return kErrUnsupported;
    if (ld % 4 != 0 || q_col % 4 != 0 || k_col % 4 != 0 || v_col % 4 != 0 || g_col % 4 != 0 || ld_out % 4 != 0 ||
        reinterpret_cast<uintptr_t>(p) % 16 != 0 || reinterpret_cast<uintptr_t>(out) % 8 != 0 || reinterpret_cast<uintptr_t>(norm_w) % 16 != 0)
        return kErrUnsupported;
    const MlstmInput in = mlstm_input(p, ld, q_col, k_col, v_col, i_col, f_col, bias, cap, q_scale, heads, dim, vdim);
    const MlstmChunks ck{add, ends, chunk_from, static_cast<bf16*>(s_hi), static_cast<bf16*>(s_lo), z, m};
    const int cpw = vdim >= 128 ? 2 : 1;
    const dim3 add_grid(n_seq * n_chunks, heads, (vdim + 64 * cpw - 1) / (64 * cpw));
#define LLME_ADD(DT)                                                                                                                \
    do {                                                                                                                            \
        if (cpw == 2) hipLaunchKernelGGL((mlstm_chunk_add_kernel<DT, 2>), add_grid, dim3(256), 0, stream, in, q_start, n_chunks, ck); \
        else hipLaunchKernelGGL((mlstm_chunk_add_kernel<DT, 1>), add_grid, dim3(256), 0, stream, in, q_start, n_chunks, ck);         \
    } while (0)
    if (dim <= 64) LLME_ADD(4);
    else if (dim <= 128) LLME_ADD(8);
    else LLME_ADD(16);
#undef LLME_ADD
    const int items = heads * (vdim + 1) * (dim / 4);
    hipLaunchKernelGGL(mlstm_chunk_carry_kernel, dim3((items + 255) / 256, n_seq), dim3(256), 0, stream, memory, level, q_start, slots, heads,
                       dim, vdim, ck);
    const int DP = dim <= 64 ? 64 : dim <= 128 ? 128 : 256;
    const int lds = 2 * (2 * 64 * (DP + 8) + vdim * 72 + 2 * 64 * 72);
    const dim3 read_grid(n_seq * n_chunks * 2, heads);
#define LLME_READ_DS(NW, NCT, DS)                                                                                                          \
    do {                                                                                                                            \
        static bool attr_set = false;                                                                                               \
        if (!attr_set) {                                                                                                            \
            const hipError_t err = hipFuncSetAttribute(reinterpret_cast<const void*>(&mlstm_chunk_read_kernel<NW, NCT, DS>),           \
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024);                     \
            if (err != hipSuccess) return static_cast<int>(err);                                                                    \
            attr_set = true;                                                                                                        \
        }                                                                                                                           \
        hipLaunchKernelGGL((mlstm_chunk_read_kernel<NW, NCT, DS>), read_grid, dim3(NW * 64), lds, stream, in, q_start, n_chunks, slots, level, ck,    \
                           norm_w, g_col, eps, scale, static_cast<bf16*>(out), ld_out);                                             \
    } while (0)
#define LLME_READ(NW, NCT)                           \
    do {                                             \
        if (dim <= 64) LLME_READ_DS(NW, NCT, 2);     \
        else if (dim <= 128) LLME_READ_DS(NW, NCT, 4); \
        else LLME_READ_DS(NW, NCT, 8);               \
    } while (0)
    if (vdim <= 64) LLME_READ(4, 1);
    else if (vdim <= 128) LLME_READ(8, 1);
    else LLME_READ(8, 2);
#undef LLME_READ
#undef LLME_READ_DS
    return launch_status();
}

LLME_LOAD_ENTRY(mlstm)
