// A matrix state per head with S_t = diag(a_t) S_(t-1) + k_t v_t^T and o_t = S_t^T q_t over a prompt, in
// chunks of 64 tokens whose work is products on the matrix cores in 32-bit (v_mfma_f32: float operands,
// float sums), so that nothing is rounded to less than a float.  a_t is a decay per row of the state and
// token (kind 1) or one number a head (kind 3).  Three kernels:
//   sums   every chunk's  N = sum_j (k_j prod_(t > j) a_t) v_j^T  and the product P of its decays
//   carry  from chunk to chunk: S_start of every chunk (in N's place), the last state to the slot
//   out    o_i = sum_(j <= i) A_ij v_j + (q_i prod_(t <= i) a_t)^T S_start,
//          A_ij = sum_c q_ic k_jc prod_(j < t <= i) a_tc
// Every factor is a product of decays, each at most one: nothing is divided by a product of decays, so
// channels that forget everything at once are as exact as the others.  With fixed decays A is q k^T times
// powers of the decay.  With decays per row the chunk is cut into blocks of 16 tokens: a pair of blocks
// I > J meets at I's first token (q_i times the decays of its own block up to i, k_j times those of its
// block behind j, times the blocks between), a product on the matrix cores; a block with itself is summed
// up lane by lane over the channels.
#include "decay_scan.h"

#include "api.h"

#define DC_LEN 64            // tokens a chunk
#define DC_SUB 16            // tokens a block

typedef __attribute__((ext_vector_type(16))) float f32x16;
typedef __attribute__((ext_vector_type(4))) float f32x4;

__device__ __forceinline__ float silu_f(float x) { return x / (1.f + expf(-x)); }

struct ChunkWork {
    int seq, chunk, head, row0, n;
    float* sums;         // [key_dim][value_dim]: N, then S_start
    float* decays;       // [key_dim]: P (kind 1)
};

__device__ __forceinline__ float* dc_sums(const DecayScan& a, int seq, int chunk, int head) {
    return a.ws + (((size_t)seq * a.chunks_per_seq + chunk) * a.heads + head) * ((size_t)a.key_dim * a.value_dim + a.key_dim);
}
// whether the workgroup's (sequence, chunk, head) has tokens
__device__ __forceinline__ bool dc_work(const DecayScan& a, int unit, ChunkWork& w) {
    w.head = unit % a.heads;
    w.chunk = unit / a.heads % a.chunks_per_seq;
    w.seq = unit / a.heads / a.chunks_per_seq;
    w.row0 = a.cu_seqlens[w.seq] + w.chunk * DC_LEN;
    w.n = min(DC_LEN, a.cu_seqlens[w.seq + 1] - w.row0);
    w.sums = dc_sums(a, w.seq, w.chunk, w.head);
    w.decays = w.sums + (size_t)a.key_dim * a.value_dim;
    return w.n > 0;
}
// first channel of the head in the rows of q and k, and a row of its decays
__device__ __forceinline__ int dc_keys(const DecayScan& a, int head) { return head / (a.heads / a.key_heads) * a.key_dim; }
__device__ __forceinline__ const float* dc_decay_row(const DecayScan& a, size_t row, int keys) {
    return (a.dt_stride > 0 ? a.dt + row * a.dt_stride + a.dt_off : a.qk + row * a.qk_stride + a.a_off) + keys;
}

// One wave per 64 key channels by 64 values of a chunk's sum: the tokens are the products' inner
// dimension, two a step, from the last to the first, so that the decays behind a token are a running
// product.  Operands come straight from memory (32 adjacent floats of two rows a load).
template <int KIND>
__global__ __launch_bounds__(WAVE) void decay_chunk_sums_kernel(DecayScan a, int quads_v, int quads) {
    ChunkWork w;
    const int quad = blockIdx.x % quads;
    if (!dc_work(a, blockIdx.x / quads, w)) return;
    const int lane = threadIdx.x, l32 = lane % 32, h = lane / 32, keys = dc_keys(a, w.head), kd = a.key_dim, vd = a.value_dim;
    const int c_base = quad / quads_v * 64, v_base = quad % quads_v * 64;
    const float fixed = KIND == 3 ? a.A[w.head] : 1.f;
    const auto read = [&](float x) { return a.act ? silu_f(x) : x; };
    f32x16 acc[2][2];
#pragma unroll
    for (int r = 0; r < 2; ++r)
#pragma unroll
        for (int q = 0; q < 2; ++q)
#pragma unroll
            for (int e = 0; e < 16; ++e) acc[r][q][e] = 0.f;
    float D[2] = {1.f, 1.f};
#pragma unroll 4
    for (int s = (w.n + 1) / 2 - 1; s >= 0; --s) {
        const int t = 2 * s + h;
        const bool there = t < w.n, second = 2 * s + 1 < w.n;
        const size_t row = w.row0 + min(t, w.n - 1);
        float A[2], B[2];
#pragma unroll
        for (int r = 0; r < 2; ++r) {
            const int c = c_base + 32 * r + l32, cc = min(c, kd - 1);
            const float k = read(a.qk[row * a.qk_stride + a.k_off + keys + cc]) * a.k_scale;
            float a0 = fixed, a1 = second ? fixed : 1.f;
            if (KIND == 1) {
                a0 = dc_decay_row(a, w.row0 + 2 * s, keys)[cc];
                a1 = second ? dc_decay_row(a, w.row0 + 2 * s + 1, keys)[cc] : 1.f;
            }
            A[r] = there && c < kd ? k * (h ? D[r] : D[r] * a1) : 0.f;
            D[r] *= a0 * a1;
        }
#pragma unroll
        for (int q = 0; q < 2; ++q) {
            const int c = v_base + 32 * q + l32;
            const float x = read(a.x[row * a.x_stride + a.x_off + (size_t)w.head * vd + min(c, vd - 1)]);
            B[q] = there && c < vd ? x : 0.f;
        }
#pragma unroll
        for (int r = 0; r < 2; ++r)
#pragma unroll
            for (int q = 0; q < 2; ++q) acc[r][q] = __builtin_amdgcn_mfma_f32_32x32x2f32(A[r], B[q], acc[r][q], 0, 0, 0);
    }
#pragma unroll
    for (int r = 0; r < 2; ++r)
#pragma unroll
        for (int q = 0; q < 2; ++q)
#pragma unroll
            for (int e = 0; e < 16; ++e) {
                const int c = c_base + 32 * r + 8 * (e >> 2) + 4 * h + (e & 3), v = v_base + 32 * q + l32;
                if (c < kd && v < vd) w.sums[(size_t)c * vd + v] = acc[r][q][e];
            }
    if (KIND == 1 && v_base == 0 && h == 0)
#pragma unroll
        for (int r = 0; r < 2; ++r)
            if (c_base + 32 * r + l32 < kd) w.decays[c_base + 32 * r + l32] = D[r];
}

// A thread an element of the state, DC_AHEAD chunks' sums on their way at a time.
#define DC_AHEAD 8
__global__ __launch_bounds__(256) void decay_chunk_carry_kernel(DecayScan a) {
    const int per_head = a.key_dim * a.value_dim;
    const int64_t e = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    const int seq = blockIdx.y;
    if (e >= (int64_t)a.heads * per_head) return;
    const int head = (int)(e / per_head), within = (int)(e % per_head), c = within / a.value_dim;
    const int n = a.cu_seqlens[seq + 1] - a.cu_seqlens[seq], n_chunks = (n + DC_LEN - 1) / DC_LEN;
    if (n_chunks == 0) return;
    float* st = a.state + (size_t)a.seq_slot[seq] * a.slot_floats + (size_t)e;
    float s = *st, whole = 1.f, rest = 1.f;      // a fixed decay over a whole chunk, and over the last one
    if (a.kind == 3) {
        const float decay = a.A[head];
        const int n_rest = n - (n_chunks - 1) * DC_LEN;
        for (int t = 0; t < DC_LEN; ++t) {
            whole *= decay;
            if (t < n_rest) rest *= decay;
        }
    }
    for (int c0 = 0; c0 < n_chunks; c0 += DC_AHEAD) {
        float sum[DC_AHEAD], decay[DC_AHEAD];
#pragma unroll
        for (int i = 0; i < DC_AHEAD; ++i) {
            const int ch = min(c0 + i, n_chunks - 1);
            const float* p = dc_sums(a, seq, ch, head);
            sum[i] = p[within];
            decay[i] = a.kind == 3 ? (ch + 1 < n_chunks ? whole : rest) : p[per_head + c];
        }
#pragma unroll
        for (int i = 0; i < DC_AHEAD; ++i) {
            if (c0 + i >= n_chunks) break;
            dc_sums(a, seq, c0 + i, head)[within] = s;
            s = decay[i] * s + sum[i];
        }
    }
    *st = s;
}

// The sums over a wave's 64 lanes of the 136 numbers that every lane holds (the pairs i >= j of a block, at
// i (i + 1) / 2 + j): each exchange halves the numbers a lane still answers for, down to three, of which
// lane l has the numbers from `first` on.
#define DC_PAIRS (DC_SUB * (DC_SUB + 1) / 2)
#define DC_PADDED 192
template <int HALF, int BIT>
__device__ __forceinline__ void halve(float (&p)[DC_PADDED], int lane, int& first) {
    const bool upper = lane & BIT;
#pragma unroll
    for (int i = 0; i < HALF; ++i) {
        const float give = upper ? p[i] : p[i + HALF], keep = upper ? p[i + HALF] : p[i];
        p[i] = keep + __shfl_xor(give, BIT, WAVE);
    }
    if (upper) first += HALF;
}

// One workgroup per (sequence, chunk, head), four waves.
template <int KIND>
__global__ __launch_bounds__(256, 2) void decay_chunk_out_kernel(DecayScan a, int ld) {
    extern __shared__ float dc_lds[];
    ChunkWork w;
    if (!dc_work(a, blockIdx.x, w)) return;
    const int kd = a.key_dim, vd = a.value_dim, kp = ld - 1, keys = dc_keys(a, w.head);
    float* Q = dc_lds;                                    // [64][ld]
    float* K = Q + DC_LEN * ld;                           // [64][ld], later A [64][65]
    float* blocks = K + DC_LEN * max(ld, DC_LEN + 1);     // kind 1: [4][kp] products of a block's decays; kind 3: powers of the decay [65]
    const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE;
    const auto read = [&](float x) { return a.act ? silu_f(x) : x; };
    float own[3] = {0.f, 0.f, 0.f};                       // kind 1: three of the wave's own block's pairs
    int own_first = 0;
    if (KIND == 3) {
        for (int idx = tid; idx < DC_LEN * kp; idx += 256) {
            const int t = idx / kp, c = idx % kp;
            const bool in = t < w.n && c < kd;
            const float* p = a.qk + (size_t)(w.row0 + min(t, w.n - 1)) * a.qk_stride + keys + min(c, kd - 1);
            const float q = read(p[a.q_off]) * a.q_scale, k = read(p[a.k_off]) * a.k_scale;
            Q[t * ld + c] = in ? q : 0.f;
            K[t * ld + c] = in ? k : 0.f;
        }
        if (tid <= DC_LEN) {
            const float decay = a.A[w.head];
            float p = 1.f;
            for (int t = 0; t < tid; ++t) p *= decay;
            blocks[tid] = p;
        }
    } else {
        float pairs[DC_PADDED];
#pragma unroll
        for (int i = 0; i < DC_PADDED; ++i) pairs[i] = 0.f;
        const int t0 = wave * DC_SUB;
        for (int c = lane; c < kp; c += WAVE) {
            float q[DC_SUB], k[DC_SUB], d[DC_SUB];
#pragma unroll
            for (int i = 0; i < DC_SUB; ++i) {
                const bool in = t0 + i < w.n && c < kd;
                const size_t row = w.row0 + min(t0 + i, w.n - 1);
                const int cc = min(c, kd - 1);
                const float* p = a.qk + row * a.qk_stride + keys + cc;
                const float qv = read(p[a.q_off]) * a.q_scale, kv = read(p[a.k_off]) * a.k_scale, dv = dc_decay_row(a, row, keys)[cc];
                q[i] = in ? qv : 0.f, k[i] = in ? kv : 0.f, d[i] = in ? dv : 1.f;
            }
            float p = 1.f;
#pragma unroll
            for (int i = 0; i < DC_SUB; ++i) {
                p *= d[i];
                Q[(t0 + i) * ld + c] = q[i] * p;
            }
            blocks[wave * kp + c] = p;
            p = 1.f;
#pragma unroll
            for (int i = DC_SUB - 1; i >= 0; --i) {
                K[(t0 + i) * ld + c] = k[i] * p;
                p *= d[i];
            }
#pragma unroll
            for (int j = 0; j < DC_SUB; ++j) {
                float kj = k[j];                              // times the decays behind j up to i
#pragma unroll
                for (int i = j; i < DC_SUB; ++i) {
                    if (i > j) kj *= d[i];
                    pairs[i * (i + 1) / 2 + j] += q[i] * kj;
                }
            }
        }
        halve<96, 32>(pairs, lane, own_first);
        halve<48, 16>(pairs, lane, own_first);
        halve<24, 8>(pairs, lane, own_first);
        halve<12, 4>(pairs, lane, own_first);
        halve<6, 2>(pairs, lane, own_first);
        halve<3, 1>(pairs, lane, own_first);
#pragma unroll
        for (int i = 0; i < 3; ++i) own[i] = pairs[i];
    }
    __syncthreads();
    // pairs of blocks: kind 3 all I >= J (ten), kind 1 all I > J (six); a wave has up to three
    constexpr int n_pairs = KIND == 3 ? 10 : 6;
    f32x4 S[3];
    int block_i[3], block_j[3];
#pragma unroll
    for (int u = 0; u < 3; ++u) {
        const int idx = wave + 4 * u;
        S[u] = {0.f, 0.f, 0.f, 0.f};
        block_i[u] = -1, block_j[u] = 0;
        if (idx >= n_pairs) continue;
        int I = 0;
        while ((I + 1) * (I + 2) / 2 <= idx) ++I;
        const int J = idx - I * (I + 1) / 2;
        const int bi = KIND == 3 ? I : I + 1;
        block_i[u] = bi, block_j[u] = J;
        const float* qp = Q + (bi * DC_SUB + lane % 16) * ld + lane / 16;
        const float* kq = K + (J * DC_SUB + lane % 16) * ld + lane / 16;
        const float* between = blocks + lane / 16;
#pragma unroll 4
        for (int c = 0; c < kp; c += 4) {
            float qv = qp[c];
            if (KIND == 1)
                for (int m = J + 1; m < bi; ++m) qv *= between[m * kp + c];
            S[u] = __builtin_amdgcn_mfma_f32_16x16x4f32(qv, kq[c], S[u], 0, 0, 0);
        }
    }
    __syncthreads();                                      // K has been read: A takes its place
    float* A = K;
    for (int idx = tid; idx < DC_LEN * (DC_LEN + 1); idx += 256) A[idx] = 0.f;
    if (KIND == 1)                                        // blocks: from a block's own product to that of all blocks before it
        for (int c = tid; c < kp; c += 256) {
            float p = 1.f;
#pragma unroll
            for (int m = 0; m < DC_LEN / DC_SUB; ++m) {
                const float mine = blocks[m * kp + c];
                blocks[m * kp + c] = p;
                p *= mine;
            }
        }
    __syncthreads();
#pragma unroll
    for (int u = 0; u < 3; ++u)
        if (block_i[u] >= 0)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int i = block_i[u] * DC_SUB + 4 * (lane / 16) + e, j = block_j[u] * DC_SUB + lane % 16;
                if (KIND == 3) A[i * (DC_LEN + 1) + j] = i >= j ? S[u][e] * blocks[max(i - j, 0)] : 0.f;
                else A[i * (DC_LEN + 1) + j] = S[u][e];
            }
    if (KIND == 1)
#pragma unroll
        for (int u = 0; u < 3; ++u) {
            const int idx = own_first + u;
            if (idx >= DC_PAIRS) continue;
            int i = 0;
            while ((i + 1) * (i + 2) / 2 <= idx) ++i;
            A[(wave * DC_SUB + i) * (DC_LEN + 1) + wave * DC_SUB + idx - i * (i + 1) / 2] = own[u];
        }
    __syncthreads();
    // outputs: tiles of 32 tokens by 32 values; a wave takes both tiles of tokens of every fourth tile of
    // values, or where there are at most two of those, one tile of tokens of one
    const int l32 = lane % 32, h = lane / 32, tiles_v = (vd + 31) / 32;
    const bool split = tiles_v <= 2;
    const float p0 = KIND == 3 ? blocks[l32 + 1] : 0.f, p1 = KIND == 3 ? blocks[33 + l32] : 0.f;
    for (int tv = split ? wave / 2 : wave; tv < tiles_v; tv += 4) {
        const bool first = !split || wave % 2 == 0, second = (!split || wave % 2 == 1) && w.n > 32;
        const int v = tv * 32 + l32, vv = min(v, vd - 1);
        f32x16 O0, O1;
#pragma unroll
        for (int e = 0; e < 16; ++e) O0[e] = 0.f, O1[e] = 0.f;
        const float *q0 = Q + l32 * ld + h, *q1 = q0 + 32 * ld;
        const float *b0 = blocks + l32 / 16 * kp + h, *b1 = b0 + 2 * kp;
        const float* sp = w.sums + vv;
#pragma unroll 8
        for (int c = 0; c < kp; c += 2) {
            const float B = c + h < kd ? sp[(size_t)min(c + h, kd - 1) * vd] : 0.f;
            if (first) O0 = __builtin_amdgcn_mfma_f32_32x32x2f32(q0[c] * (KIND == 3 ? p0 : b0[c]), B, O0, 0, 0, 0);
            if (second) O1 = __builtin_amdgcn_mfma_f32_32x32x2f32(q1[c] * (KIND == 3 ? p1 : b1[c]), B, O1, 0, 0, 0);
        }
        const float *a0 = A + l32 * (DC_LEN + 1) + h, *a1 = a0 + 32 * (DC_LEN + 1);
        const float* xp = a.x + (size_t)w.row0 * a.x_stride + a.x_off + (size_t)w.head * vd + vv;
#pragma unroll 8
        for (int j = 0; j < 32; j += 2) {
            const float x = read(xp[(size_t)min(j + h, w.n - 1) * a.x_stride]), B = j + h < w.n ? x : 0.f;
            if (first) O0 = __builtin_amdgcn_mfma_f32_32x32x2f32(a0[j], B, O0, 0, 0, 0);
            if (second) O1 = __builtin_amdgcn_mfma_f32_32x32x2f32(a1[j], B, O1, 0, 0, 0);
        }
        if (second)
#pragma unroll 8
            for (int j = 32; j < DC_LEN; j += 2) {
                const float x = read(xp[(size_t)min(j + h, w.n - 1) * a.x_stride]), B = j + h < w.n ? x : 0.f;
                O1 = __builtin_amdgcn_mfma_f32_32x32x2f32(a1[j], B, O1, 0, 0, 0);
            }
        float* out = a.out + ((size_t)w.row0 * a.heads + w.head) * vd + v;
        const size_t out_stride = (size_t)a.heads * vd;
        if (v < vd)
#pragma unroll
            for (int e = 0; e < 16; ++e) {
                const int i = 8 * (e >> 2) + 4 * h + (e & 3);
                if (first && i < w.n) out[i * out_stride] = O0[e];
                if (second && i + 32 < w.n) out[(i + 32) * out_stride] = O1[e];
            }
    }
}

size_t picolm_decay_chunks_ws_floats(const DecayScan& a, int n_seq, int most_new) {
    return (size_t)n_seq * ceil_div(most_new, DC_LEN) * a.heads * ((size_t)a.key_dim * a.value_dim + a.key_dim);
}

int picolm_decay_chunks(DecayScan a, int n_seq, int most_new, hipStream_t stream) {
    PICOLM_REQUIRE((a.kind == 1 || a.kind == 3) && !a.skip && a.ws && a.key_dim <= 256, "decay_chunks: kind %d, keys of %d", a.kind, a.key_dim);
    a.chunks_per_seq = ceil_div(most_new, DC_LEN);
    const int64_t units = (int64_t)n_seq * a.chunks_per_seq * a.heads;
    const int quads_v = ceil_div(a.value_dim, 64), quads = ceil_div(a.key_dim, 64) * quads_v;
    PICOLM_REQUIRE(units * quads < (1ll << 31) && n_seq <= 65535, "decay_chunks: %lld chunks exceed the grid", (long long)units);
    const dim3 sums((unsigned)(units * quads));
    if (a.kind == 3) decay_chunk_sums_kernel<3><<<sums, WAVE, 0, stream>>>(a, quads_v, quads);
    else decay_chunk_sums_kernel<1><<<sums, WAVE, 0, stream>>>(a, quads_v, quads);
    PICOLM_LAUNCH_CHECK("decay_chunks (sums)");
    const int64_t elements = (int64_t)a.heads * a.key_dim * a.value_dim;
    decay_chunk_carry_kernel<<<dim3((unsigned)ceil_div64(elements, 256), n_seq), 256, 0, stream>>>(a);
    PICOLM_LAUNCH_CHECK("decay_chunks (carry)");
    const int kp = (a.key_dim + 3) / 4 * 4, ld = kp + 1;
    const size_t lds = sizeof(float) * ((size_t)DC_LEN * (ld + (ld > DC_LEN + 1 ? ld : DC_LEN + 1)) + (4 * kp > DC_LEN + 1 ? 4 * kp : DC_LEN + 1));
    static size_t raised = 48 * 1024;      // what a kernel may use without asking
    if (lds > raised) {
        hipError_t e = hipFuncSetAttribute((const void*)decay_chunk_out_kernel<3>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e == hipSuccess) e = hipFuncSetAttribute((const void*)decay_chunk_out_kernel<1>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        PICOLM_REQUIRE(e == hipSuccess, "decay_chunks: cannot raise the LDS limit to %zu: %s", lds, hipGetErrorString(e));
        raised = lds;
    }
    if (a.kind == 3) decay_chunk_out_kernel<3><<<(unsigned)units, 256, lds, stream>>>(a, ld);
    else decay_chunk_out_kernel<1><<<(unsigned)units, 256, lds, stream>>>(a, ld);
    PICOLM_LAUNCH_CHECK("decay_chunks (out)");
    return 0;
}
