// Linear attention between its projections (mixers.h, picolm_call_linear_attention).  A prompt runs the
// operations it consists of; a decode step runs one kernel, in which a workgroup has a sequence's
// head: it turns q and k by the token's position, makes the token's decays, carries the state over the
// token, reads it out along q, and norms and gates the head's output.  All arithmetic is float; the
// state is read and written once.
#include "mixers.h"

#include "api.h"
#include "common.h"

#define VIEW_REQUIRE(who, v)                                                                                      \
    PICOLM_REQUIRE((v) && (v)->struct_bytes == (int32_t)sizeof(picolm_step_view), "%s: the step view is of another version", who)

__device__ __forceinline__ float silu_f(float x) { return x / (1.f + expf(-x)); }
__device__ __forceinline__ float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }

#define LS_THREADS 512
#define LS_ROWS 8        // rows of the state that a thread has on their way from memory at a time

struct LinearStep {
    const float* in;
    void* out;
    float* y;                // not null: the head's raw output goes here, and norm and gate follow in another kernel
    float* state;
    const int32_t* seq_slot;
    const int32_t* tok_pos;
    int64_t slot_floats;
    int columns;             // threads side by side along a row of the state, a power of two
    picolm_linear_attention_args a;
};

// A thread has VEC adjacent columns of every row i, i + groups, i + 2 groups, ... of the state.
template <typename T, int VEC>
__global__ __launch_bounds__(LS_THREADS) void linear_step_kernel(LinearStep s) {
    extern __shared__ float ls_lds[];      // q [kd] | k [kd] | decays [kd] | v [vd] | partial sums [groups][columns VEC]
    __shared__ float scratch[16];
    const picolm_decay_scan_args& sc = s.a.scan;
    const int kd = sc.key_dim, vd = sc.value_dim, head = blockIdx.x, seq = blockIdx.y, tid = threadIdx.x;
    const int columns = s.columns, groups = LS_THREADS / columns, col = (tid % columns) * VEC, group = tid / columns;
    float *qs = ls_lds, *ks = qs + kd, *as = ks + kd, *vs = as + kd, *part = vs + vd;
    const float* row = s.in + (size_t)seq * sc.x_stride;
    float* st = s.state + (size_t)s.seq_slot[seq] * s.slot_floats + (size_t)head * kd * vd;
    typedef float vec __attribute__((ext_vector_type(VEC)));
    // the first rows of the state are asked for before anything else
    vec S[LS_ROWS];
    auto load = [&](int c, int r0) {
#pragma unroll
        for (int i = 0; i < LS_ROWS; ++i) {
            const int r = r0 + i * groups;
            if (r < kd && c < vd) S[i] = *(const vec*)(st + (size_t)r * vd + c);
        }
    };
    load(col, group);
    const auto read = [&](float x) { return sc.act ? silu_f(x) : x; };
    const int half = s.a.rot_dims / 2;
    const size_t table_row = s.a.cos_table ? (size_t)min(s.tok_pos[seq], s.a.table_positions - 1) * half : 0;
    for (int i = tid; i < kd; i += LS_THREADS) {
        const float *q = row + sc.q_off + head * kd, *k = row + sc.k_off + head * kd;
        float qv = read(q[i]), kv = read(k[i]);
        if (s.a.cos_table && i < s.a.rot_dims) {
            const bool first = s.a.rot_half ? i < half : (i & 1) == 0;
            const int j = s.a.rot_half ? (first ? i : i - half) : i >> 1, other = s.a.rot_half ? (first ? i + half : i - half) : i ^ 1;
            const float c = s.a.cos_table[table_row + j], sn = first ? -s.a.sin_table[table_row + j] : s.a.sin_table[table_row + j];
            qv = qv * c + q[other] * sn;
            kv = kv * c + k[other] * sn;
        }
        qs[i] = qv * sc.q_scale;
        ks[i] = kv * sc.k_scale;
        float decay;
        if (sc.kind == 3) {
            decay = sc.A[head];
        } else {
            const picolm_channel_decays_args& d = s.a.decays;
            const int ch = head * kd + i;
            float z = d.bias ? d.bias[ch] : 0.f;
#pragma unroll 8
            for (int r = 0; r < d.rank; ++r) z = fmaf(d.weight[(size_t)r * d.channels + ch], row[d.in_off + r], z);
            const float n = -z, sp = n > 20.f ? n : log1pf(expf(n));
            decay = expf(-d.power * sp);
        }
        as[i] = decay;
    }
    for (int i = tid; i < vd; i += LS_THREADS) vs[i] = read(row[sc.x_off + head * vd + i]);
    __syncthreads();
    const picolm_gated_norm_args& n = s.a.norm;
    const float* gate = row + n.gate_off + (size_t)head * vd;
    float ssq = 0.f;
    for (int c0 = 0; c0 < vd; c0 += columns * VEC) {
        const int c = c0 + col;
        vec acc, v;
#pragma unroll
        for (int j = 0; j < VEC; ++j) acc[j] = 0.f, v[j] = c + j < vd ? vs[c + j] : 0.f;
        for (int r0 = group; r0 < kd; r0 += LS_ROWS * groups) {
            if (c0 > 0 || r0 > group) load(c, r0);
#pragma unroll
            for (int i = 0; i < LS_ROWS; ++i) {
                const int r = r0 + i * groups;
                if (r < kd && c < vd) {
                    const float a = as[r], k = ks[r], q = qs[r];
#pragma unroll
                    for (int j = 0; j < VEC; ++j) {
                        S[i][j] = a * S[i][j] + k * v[j];
                        acc[j] += q * S[i][j];
                    }
                    *(vec*)(st + (size_t)r * vd + c) = S[i];
                }
            }
        }
#pragma unroll
        for (int j = 0; j < VEC; ++j) part[group * columns * VEC + col + j] = acc[j];
        __syncthreads();
        for (int i = tid; i < columns * VEC; i += LS_THREADS) {
            float o = 0.f;
            for (int g = 0; g < groups; ++g) o += part[g * columns * VEC + i];
            if (c0 + i < vd) {
                vs[c0 + i] = o;             // (the value has been read by then: the columns of this round only)
                ssq += o * o;
            }
        }
        __syncthreads();
    }
    if (s.y) {
        for (int i = tid; i < vd; i += LS_THREADS) s.y[((size_t)seq * sc.n_heads + head) * vd + i] = vs[i];
        return;
    }
    const float inv = 1.f / sqrtf(block_sum(ssq, scratch) / (float)vd + n.eps);
    const int out_stride = n.out_stride ? n.out_stride : n.width;
    T* out = (T*)s.out + (size_t)seq * out_stride + n.out_off + (size_t)head * vd;
    const float mult = n.out_stride ? n.mult : 1.f;
    for (int i = tid; i < vd; i += LS_THREADS) {
        float o = vs[i] * inv * (n.weight ? n.weight[i] : 1.f);
        o *= n.gate_act == 2 ? sigmoid_f(gate[i]) : silu_f(gate[i]);
        out[i] = from_f32<T>(o * mult);
    }
}

extern "C" int picolm_call_linear_attention(void* user, const picolm_step_view* v) {
    picolm_linear_attention_args* a = (picolm_linear_attention_args*)user;
    VIEW_REQUIRE("linear_attention", v);
    PICOLM_REQUIRE(a && v->in && v->out && v->extra[0], "linear_attention: buffers are missing");
    picolm_decay_scan_args& sc = a->scan;
    const bool made = a->decays.weight != nullptr;
    PICOLM_REQUIRE(sc.kind == (made ? 1 : 3) && sc.n_heads == sc.n_key_heads && !sc.skip && (!made || (v->extra[1] && sc.dt_stride == a->decays.channels && sc.dt_off == 0)),
                   "linear_attention: fixed decays, or decays that it makes itself, with a key head a head");
    PICOLM_REQUIRE(sc.qk_stride == sc.x_stride && a->norm.gate_stride == sc.x_stride && (!made || a->decays.in_stride == sc.x_stride) &&
                       a->norm.width == sc.n_heads * sc.value_dim && !a->norm.gate_first,
                   "linear_attention: the operations' rows differ");
    PICOLM_REQUIRE(!a->cos_table || (a->sin_table && a->table_positions > 0 && a->rot_dims > 0 && a->rot_dims % 2 == 0 && a->rot_dims <= sc.key_dim &&
                                     !sc.act && v->tok_pos && v->rows == v->n_tokens),
                   "linear_attention: a rotation of %d entries of %d, tables for %d positions (it takes no activation)", a->rot_dims, sc.key_dim,
                   a->table_positions);
    if (v->n_tokens <= 0) return 0;
    if (a->cos_table)
        for (int i = 0; i < v->n_seq; ++i)
            PICOLM_REQUIRE(v->recording || v->pos0[i] + v->n_new[i] <= a->table_positions,
                           "linear_attention: sequence %d reaches position %d, the tables hold %d", i, v->pos0[i] + v->n_new[i], a->table_positions);
    picolm_step_view w = *v;
    const auto give = [&](void* in, int in_bytes, void* out, int out_bytes, void* e0, int e0_bytes, void* e1, int e1_bytes) {
        w.in = in, w.in_row_bytes = in_bytes, w.out = out, w.out_row_bytes = out_bytes;
        w.extra[0] = e0, w.extra_row_bytes[0] = e0_bytes, w.extra[1] = e1, w.extra_row_bytes[1] = e1_bytes;
    };
    const auto norm = [&]() {
        give(v->extra[0], v->extra_row_bytes[0], v->out, v->out_row_bytes, v->in, v->in_row_bytes, nullptr, 0);
        return picolm_call_gated_norm(&a->norm, &w);
    };
    if (!v->is_decode) {
        if (a->cos_table) {       // q and k in place: one pass where their heads lie side by side
            picolm_rotate_heads_args r = {};
            const bool joined = sc.k_off == sc.q_off + sc.n_heads * sc.key_dim;
            r.cos_table = a->cos_table, r.sin_table = a->sin_table, r.table_positions = a->table_positions;
            r.dims = a->rot_dims, r.half = a->rot_half, r.heads = sc.n_heads * (joined ? 2 : 1), r.width = a->rot_dims;
            r.in_stride = r.out_stride = sc.qk_stride, r.in_head_stride = r.out_head_stride = sc.key_dim;
            give(v->in, v->in_row_bytes, v->in, v->in_row_bytes, nullptr, 0, nullptr, 0);
            r.in_off = r.out_off = sc.q_off;
            if (const int rc = picolm_call_rotate_heads(&r, &w)) return rc;
            r.in_off = r.out_off = sc.k_off;
            if (!joined)
                if (const int rc = picolm_call_rotate_heads(&r, &w)) return rc;
        }
        if (made) {
            give(v->in, v->in_row_bytes, v->extra[1], v->extra_row_bytes[1], nullptr, 0, nullptr, 0);
            if (const int rc = picolm_call_channel_decays(&a->decays, &w)) return rc;
        }
        give(v->in, v->in_row_bytes, v->extra[0], v->extra_row_bytes[0], v->in, v->in_row_bytes, made ? v->extra[1] : nullptr,
             made ? v->extra_row_bytes[1] : 0);
        if (const int rc = picolm_call_decay_scan(&sc, &w)) return rc;
        return norm();
    }
    // a decode step: every row is a sequence
    const int heads = sc.n_heads, kd = sc.key_dim, vd = sc.value_dim;
    const int es = v->dtype == PICOLM_F32 ? 4 : 2, out_stride = a->norm.out_stride ? a->norm.out_stride : a->norm.width;
    PICOLM_REQUIRE(heads > 0 && kd > 0 && kd <= 256 && vd > 0 && v->n_seq == v->n_tokens && heads <= (1 << 30) && v->n_seq <= 65535,
                   "linear_attention: %d heads with keys of %d and values of %d, %d sequences", heads, kd, vd, v->n_seq);
    PICOLM_REQUIRE(sc.q_off >= 0 && sc.q_off + heads * kd <= sc.x_stride && sc.k_off >= 0 && sc.k_off + heads * kd <= sc.x_stride && sc.x_off >= 0 &&
                       sc.x_off + heads * vd <= sc.x_stride && a->norm.gate_off >= 0 && a->norm.gate_off + heads * vd <= sc.x_stride &&
                       (!made || (a->decays.channels == heads * kd && a->decays.rank > 0 && a->decays.in_off >= 0 &&
                                  a->decays.in_off + a->decays.rank <= sc.x_stride)) &&
                       v->in_row_bytes >= (int64_t)sc.x_stride * 4 && v->extra_row_bytes[0] >= heads * vd * 4,
                   "linear_attention: rows of %d floats do not hold what the offsets name", sc.x_stride);
    PICOLM_REQUIRE(made || sc.A, "linear_attention: fixed decays are missing");
    PICOLM_REQUIRE((a->norm.out_stride > 0 || a->norm.out_off == 0) && a->norm.out_off >= 0 && a->norm.out_off + a->norm.width <= out_stride &&
                       v->out_row_bytes >= (int64_t)out_stride * es && (a->norm.group == vd || a->norm.group == a->norm.width),
                   "linear_attention: output rows too short, or a norm over neither a head nor all of them");
    PICOLM_REQUIRE(!a->norm.weight || a->norm.weight_len == a->norm.group, "linear_attention: a norm's weight of another size than what it norms");
    const int64_t need = (sc.state_off + (int64_t)heads * kd * vd) * 4;
    PICOLM_REQUIRE(v->state && sc.state_off >= 0 && need <= v->state_bytes_per_slot, "linear_attention: the state of a slot has %lld bytes, the matrices need %lld",
                   (long long)v->state_bytes_per_slot, (long long)need);
    const bool joint = a->norm.group != vd;
    LinearStep s;
    s.in = (const float*)v->in, s.out = v->out, s.y = joint ? (float*)v->extra[0] : nullptr;
    s.state = (float*)v->state + sc.state_off, s.seq_slot = v->seq_slot, s.tok_pos = v->tok_pos, s.slot_floats = v->state_bytes_per_slot / 4;
    s.a = *a;
    if (s.a.scan.q_scale == 0.f) s.a.scan.q_scale = 1.f;
    if (s.a.scan.k_scale == 0.f) s.a.scan.k_scale = 1.f;
    const bool wide = vd % 4 == 0 && ((uintptr_t)s.state & 15) == 0 && s.slot_floats % 4 == 0;
    const int vec = wide ? 4 : 1;
    int columns = 1;
    while (columns * vec < vd && columns < LS_THREADS) columns *= 2;
    s.columns = columns;
    const size_t lds = sizeof(float) * ((size_t)3 * kd + vd + LS_THREADS * vec);
    PICOLM_REQUIRE(lds <= 64 * 1024, "linear_attention: values of %d need %zu bytes of LDS", vd, lds);
    const dim3 grid(heads, v->n_seq);
    if (v->dtype == PICOLM_F32) {
        if (wide) linear_step_kernel<float, 4><<<grid, LS_THREADS, lds, v->stream>>>(s);
        else linear_step_kernel<float, 1><<<grid, LS_THREADS, lds, v->stream>>>(s);
    } else {
        if (wide) linear_step_kernel<bf16_t, 4><<<grid, LS_THREADS, lds, v->stream>>>(s);
        else linear_step_kernel<bf16_t, 1><<<grid, LS_THREADS, lds, v->stream>>>(s);
    }
    PICOLM_LAUNCH_CHECK("linear_attention (step)");
    return joint ? norm() : 0;
}
