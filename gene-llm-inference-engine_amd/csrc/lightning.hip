// Linear attention whose memory fades by a constant per head ("lightning" attention), in 32-bit.
//
// Per head, with d the head's decay, q = SiLU(q'), k = SiLU(k'), v = SiLU(v') of the projected rows, and S [dk][dv] zero at a
// sequence's start:
//     S_t = d S_(t-1) + k_t v_t^T         o_t = S_t^T q_t
// State of one request slot: [head][dk][dv], 32-bit.
//
// Two forms.  Token by token (`lightning_scan_kernel`): columns of S never meet, so a workgroup owns 16 columns of one head of one
// request and walks the request's rows in order; every sum's order is fixed by dk alone, so the bits do not depend on how the rows
// were cut into steps.  In chunks of 64 rows that run at once, on the 32-bit matrix instructions (three kernels): what a chunk alone
// leaves in S, U = sum_t d^(n-1-t) k_t v_t^T over its n rows; the states the chunks start from, S <- d^n S + U from chunk to
// chunk; and the rows' results,
//     o_i = d^(i+1) S^T q_i + sum_(j <= i) d^(i-j) (q_i . k_j) v_j      (i, j counted in the chunk, S the state it starts from).
// The powers of every head's decay come in a table [heads][65], d^0 .. d^64, made on the host in 64-bit.
#include "common.h"

namespace {

typedef float floatx16 __attribute__((ext_vector_type(16)));

constexpr int CHUNK = 64;                  // rows of a chunk
constexpr int POWERS = CHUNK + 1;          // entries of a head's table of powers
constexpr int SCAN_COLS = 16;              // columns of S that a workgroup of the token-by-token kernel owns
constexpr int SCAN_GROUPS = 16;            // groups of rows its 256 threads form
constexpr int SCAN_TOKENS = 8;             // tokens staged at a time

__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
// The same by the hardware's exp2 and reciprocal (a unit or two in the last place).
__device__ __forceinline__ float silu_quick(float z) { return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z)); }

// ------------------------------------------------------------------------------------------------ token by token
// Thread = (column c, group g of rows): it keeps the rows g, g + 16, g + 32, ... of its column in registers.  A block of tokens' q and
// k (zero beyond dk) and v lie in LDS; a token's result is the thread's share over its rows, added over the wave's four groups by lane
// moves and over the four waves through LDS, once for the whole block of tokens.
template <int ROWS>
__global__ __launch_bounds__(256) void lightning_scan_kernel(const float* __restrict__ proj, long ld, int q_off, int k_off, int v_off,
                                                            const float* __restrict__ powers, const int* __restrict__ seg_start, const int* __restrict__ seg_len,
                                                            const int* __restrict__ row_slot, float* __restrict__ state, long state_stride,
                                                            float* __restrict__ out, long ldo, int dk, int dv) {
    constexpr int KQ = SCAN_GROUPS * ROWS;
    __shared__ float2 kq_s[SCAN_TOKENS][KQ];
    __shared__ float v_s[SCAN_TOKENS][SCAN_COLS];
    __shared__ float part[SCAN_TOKENS][4][SCAN_COLS];
    const int n = seg_len[blockIdx.x];
    if (n <= 0) return;                                           // (the same for the whole workgroup)
    const int t0 = seg_start[blockIdx.x], h = blockIdx.y, tid = threadIdx.x, c = tid % SCAN_COLS, g = tid / SCAN_COLS, wave = tid >> 6;
    const int col = blockIdx.z * SCAN_COLS + c;
    const int col_in = min(col, dv - 1);                          // (idle columns walk along on the last one and store nothing)
    float* st = state + (size_t)row_slot[t0] * state_stride + (size_t)h * dk * dv;
    float S[ROWS];
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
        const int i = g + SCAN_GROUPS * r;
        S[r] = i < dk ? st[(size_t)i * dv + col_in] : 0.f;
    }
    const float decay = powers[h * POWERS + 1];
    for (int b0 = 0; b0 < n; b0 += SCAN_TOKENS) {
        const int here = min(SCAN_TOKENS, n - b0);
        for (int e = tid; e < here * KQ; e += 256) {
            const int u = e / KQ, i = e % KQ;
            const float* row = proj + (size_t)(t0 + b0 + u) * ld;
            kq_s[u][i] = i < dk ? float2{silu_f(row[k_off + h * dk + i]), silu_f(row[q_off + h * dk + i])} : float2{0.f, 0.f};
        }
        if (tid < here * SCAN_COLS) v_s[tid / SCAN_COLS][c] = silu_f(proj[(size_t)(t0 + b0 + tid / SCAN_COLS) * ld + v_off + h * dv + col_in]);
        __syncthreads();
        for (int u = 0; u < here; ++u) {
            const float v = v_s[u][c];
            float acc = 0.f;
#pragma unroll
            for (int r = 0; r < ROWS; ++r) {
                const float2 kq = kq_s[u][g + SCAN_GROUPS * r];
                S[r] = fmaf(decay, S[r], kq.x * v);
                acc = fmaf(S[r], kq.y, acc);
            }
            acc += __shfl_xor(acc, 16, 64);
            acc += __shfl_xor(acc, 32, 64);
            if ((g & 3) == 0) part[u][wave][c] = acc;
        }
        __syncthreads();
        if (tid < here * SCAN_COLS && col < dv) {
            const int u = tid / SCAN_COLS;
            out[(size_t)(t0 + b0 + u) * ldo + h * dv + col] = (part[u][0][c] + part[u][1][c]) + (part[u][2][c] + part[u][3][c]);
        }
    }
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
        const int i = g + SCAN_GROUPS * r;
        if (i < dk && col < dv) st[(size_t)i * dv + col] = S[r];
    }
}

// ------------------------------------------------------------------------------------------------ in chunks
struct Chunk {
    int t0, rows;                          // first row in the step, number of rows (0: there is no such chunk)
};

// Chunk number `index` of the step: the requests' runs, each cut into chunks of CHUNK rows (the last one shorter), one after the other.
__device__ __forceinline__ Chunk find_chunk(const int* __restrict__ seg_start, const int* __restrict__ seg_len, int n_segs, int index) {
    for (int s = 0; s < n_segs; ++s) {
        const int n = seg_len[s], chunks = (n + CHUNK - 1) / CHUNK;
        if (index < chunks) return Chunk{seg_start[s] + index * CHUNK, min(CHUNK, n - index * CHUNK)};
        index -= chunks;
    }
    return Chunk{0, 0};
}

// What a chunk alone leaves in the memory: U[i][c] = sum_t d^(rows-1-t) k_t[i] v_t[c].  A wave makes one tile of 32 x 32 with 32
// instructions of 32 x 32 x 2: lane l brings row l % 32 of k^T and column l % 32 of v at the tokens 2 s + l / 32.
__global__ __launch_bounds__(256) void lightning_chunk_states_kernel(const float* __restrict__ proj, long ld, int k_off, int v_off, const float* __restrict__ powers,
                                                                    const int* __restrict__ seg_start, const int* __restrict__ seg_len, int n_segs,
                                                                    float* __restrict__ states, int n_heads, int dk, int dv) {
    const Chunk ch = find_chunk(seg_start, seg_len, n_segs, blockIdx.x);
    const int h = blockIdx.y, lane = threadIdx.x & 63, half = lane >> 5, l = lane & 31;
    const int col_tiles = (dv + 31) / 32, tile = blockIdx.z * 4 + (threadIdx.x >> 6);
    const int i0 = tile / col_tiles * 32, c0 = tile % col_tiles * 32;
    if (ch.rows <= 0 || i0 >= dk) return;
    const float* kp = proj + (size_t)ch.t0 * ld + k_off + h * dk + min(i0 + l, dk - 1);
    const float* vp = proj + (size_t)ch.t0 * ld + v_off + h * dv + min(c0 + l, dv - 1);
    const float* pw = powers + h * POWERS;
    floatx16 acc = {};
    const int steps = (ch.rows + 1) / 2;
    for (int s0 = 0; s0 < steps; s0 += 8) {
        float a[8], b[8], w[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) {                             // (rows behind the chunk's last are read as its last and weigh nothing)
            const int t = 2 * (s0 + u) + half, tc = min(t, ch.rows - 1);
            a[u] = kp[(size_t)tc * ld], b[u] = vp[(size_t)tc * ld];
            w[u] = t < ch.rows ? pw[ch.rows - 1 - tc] : 0.f;
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(silu_quick(a[u]) * w[u], silu_quick(b[u]), acc, 0, 0, 0);
    }
    if (c0 + l >= dv) return;
    float* to = states + (((size_t)blockIdx.x * n_heads + h) * dk) * dv + c0 + l;
#pragma unroll
    for (int e = 0; e < 16; ++e) {
        const int i = i0 + 8 * (e / 4) + 4 * half + (e & 3);
        if (i < dk) to[(size_t)i * dv] = acc[e];
    }
}

// From chunk to chunk of one request, a number of S a thread: `states` holds what every chunk alone leaves and gets what it starts
// from; the request's slot gets what the last one leaves.
__global__ __launch_bounds__(256) void lightning_carry_kernel(const float* __restrict__ powers, const int* __restrict__ seg_start, const int* __restrict__ seg_len,
                                                             const int* __restrict__ row_slot, float* __restrict__ state, long state_stride,
                                                             float* __restrict__ states, int n_heads, int per_head) {
    const int n = seg_len[blockIdx.x], h = blockIdx.y, e = blockIdx.z * 256 + threadIdx.x;
    if (n <= 0 || e >= per_head) return;
    int first = 0;
    for (int s = 0; s < (int)blockIdx.x; ++s) first += (seg_len[s] + CHUNK - 1) / CHUNK;
    const int chunks = (n + CHUNK - 1) / CHUNK;
    const float whole = powers[h * POWERS + CHUNK], last = powers[h * POWERS + (n - (chunks - 1) * CHUNK)];
    float* mine = state + (size_t)row_slot[seg_start[blockIdx.x]] * state_stride + (size_t)h * per_head + e;
    float* at = states + ((size_t)first * n_heads + h) * per_head + e;
    const size_t stride = (size_t)n_heads * per_head;
    constexpr int AHEAD = 8;                                      // chunks whose numbers are asked for at once
    float S = *mine;
    for (int g0 = 0; g0 < chunks; g0 += AHEAD) {
        float u[AHEAD];
#pragma unroll
        for (int j = 0; j < AHEAD; ++j) u[j] = at[(size_t)min(g0 + j, chunks - 1) * stride];
#pragma unroll
        for (int j = 0; j < AHEAD; ++j) {
            if (g0 + j < chunks) {
                at[(size_t)(g0 + j) * stride] = S;
                S = fmaf(g0 + j + 1 < chunks ? whole : last, S, u[j]);
            }
        }
    }
    *mine = S;
}

// The rows' results.  A workgroup: one chunk, one head, 64 columns of v; its four waves own the four tiles of 32 rows x 32 columns.
// Over blocks of 32 key channels q and k lie in LDS: the waves gather q S (S straight from memory) and three of them the tiles of the
// rows' weights q k^T on and under the diagonal, which go through LDS, faded, into the product with v.
constexpr int KB = 32, QS_STRIDE = KB + 1, PS_STRIDE = CHUNK + 1;
__global__ __launch_bounds__(256) void lightning_chunk_rows_kernel(const float* __restrict__ proj, long ld, int q_off, int k_off, int v_off,
                                                                  const float* __restrict__ powers, const int* __restrict__ seg_start,
                                                                  const int* __restrict__ seg_len, int n_segs, const float* __restrict__ states,
                                                                  float* __restrict__ out, long ldo, int n_heads, int dk, int dv) {
    __shared__ float q_s[CHUNK][QS_STRIDE], k_s[CHUNK][QS_STRIDE], p_s[CHUNK][PS_STRIDE], pw_s[POWERS];
    const Chunk ch = find_chunk(seg_start, seg_len, n_segs, blockIdx.x);
    if (ch.rows <= 0) return;                                     // (the same for the whole workgroup)
    const int h = blockIdx.y, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, half = lane >> 5, l = lane & 31;
    const int rt = wave & 1, ct = wave >> 1;                      // this wave's tile of the results: rows 32 rt .., columns 32 ct ..
    const int pt = wave == 3 ? 1 : 0;                             // ... and of the weights: (rt, pt); the tile (0, 1) lies above the diagonal
    const bool weighs = wave != 2;
    const int c = blockIdx.z * 64 + 32 * ct + l, cc = min(c, dv - 1);
    const float* rows = proj + (size_t)ch.t0 * ld;
    const float* S = states + (((size_t)blockIdx.x * n_heads + h) * dk) * dv + cc;
    if (tid < POWERS) pw_s[tid] = powers[h * POWERS + tid];
    floatx16 acc = {}, weights = {};
    for (int k0 = 0; k0 < dk; k0 += KB) {
        float sv[KB / 2];
#pragma unroll
        for (int s = 0; s < KB / 2; ++s) sv[s] = S[(size_t)min(k0 + 2 * s + half, dk - 1) * dv];
        if (k0) __syncthreads();                                  // the block before has been read
#pragma unroll
        for (int e = 0; e < CHUNK * KB / 256; ++e) {
            const int t = (tid + 256 * e) / KB, i = k0 + (tid + 256 * e) % KB;
            const float* row = rows + (size_t)min(t, ch.rows - 1) * ld + h * dk + min(i, dk - 1);
            const bool there = t < ch.rows && i < dk;
            q_s[t][i - k0] = there ? silu_quick(row[q_off]) : 0.f;
            k_s[t][i - k0] = there ? silu_quick(row[k_off]) : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int s = 0; s < KB / 2; ++s) {
            const float q = q_s[32 * rt + l][2 * s + half];
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(q, sv[s], acc, 0, 0, 0);
            if (weighs) weights = __builtin_amdgcn_mfma_f32_32x32x2f32(q, k_s[32 * pt + l][2 * s + half], weights, 0, 0, 0);
        }
    }
#pragma unroll
    for (int e = 0; e < 16; ++e) {
        const int i = 32 * rt + 8 * (e / 4) + 4 * half + (e & 3), j = 32 * pt + l;
        acc[e] *= pw_s[i + 1];
        if (weighs) p_s[i][j] = j <= i ? weights[e] * pw_s[i - j] : 0.f;
    }
    const float* vp = rows + v_off + h * dv + cc;
    const int steps = 16 * (rt + 1);                              // the tokens up to this tile's last row
    float v[16];
#pragma unroll
    for (int s = 0; s < 16; ++s) v[s] = vp[(size_t)min(2 * s + half, ch.rows - 1) * ld];
    __syncthreads();
    for (int s0 = 0; s0 < steps; s0 += 16) {
#pragma unroll
        for (int s = 0; s < 16; ++s) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(p_s[32 * rt + l][2 * (s0 + s) + half], silu_quick(v[s]), acc, 0, 0, 0);
        if (s0 + 16 < steps) {
#pragma unroll
            for (int s = 0; s < 16; ++s) v[s] = vp[(size_t)min(2 * (s0 + 16 + s) + half, ch.rows - 1) * ld];
        }
    }
    if (c >= dv) return;
#pragma unroll
    for (int e = 0; e < 16; ++e) {
        const int i = 32 * rt + 8 * (e / 4) + 4 * half + (e & 3);
        if (i < ch.rows) out[(size_t)(ch.t0 + i) * ldo + h * dv + c] = acc[e];
    }
}

// ------------------------------------------------------------------------------------------------ norm over the row, gate
// y[t] = w * o[t] * rsqrt(mean(o[t]^2) + eps) * sigmoid(g[t]), the mean over the whole row; a workgroup a row.  NV > 0: rows whose length
// is a multiple of 4 and at most 1024 NV, aligned: a thread asks for all its numbers at once and keeps them.
__device__ __forceinline__ float4 load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 load4(const bf16_t* p) {
    const uint2 v = *reinterpret_cast<const uint2*>(p);
    return float4{__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u), __uint_as_float(v.y << 16), __uint_as_float(v.y & 0xffff0000u)};
}
__device__ __forceinline__ void store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void store4(bf16_t* p, float4 v) { *reinterpret_cast<uint2*>(p) = uint2{f32x2_to_bf16x2(v.x, v.y), f32x2_to_bf16x2(v.z, v.w)}; }
__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }

template <int NV, typename TW, typename TO>
__global__ __launch_bounds__(256) void row_norm_gate_kernel(const float* __restrict__ o, long ldo, const float* __restrict__ g, long ldg, const TW* __restrict__ w,
                                                           TO* __restrict__ y, long ldy, int dim, float eps) {
    __shared__ float red[4];
    const float* orow = o + (size_t)blockIdx.x * ldo;
    const float* grow = g + (size_t)blockIdx.x * ldg;
    TO* yrow = y + (size_t)blockIdx.x * ldy;
    if constexpr (NV > 0) {
        float4 ov[NV], gv[NV], wv[NV];
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int d = min(4 * ((int)threadIdx.x + 256 * i), dim - 4);
            ov[i] = load4(orow + d), gv[i] = load4(grow + d), wv[i] = load4(w + d);
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const float s = (ov[i].x * ov[i].x + ov[i].y * ov[i].y) + (ov[i].z * ov[i].z + ov[i].w * ov[i].w);
            ss += 4 * ((int)threadIdx.x + 256 * i) < dim ? s : 0.f;
        }
        const float r = 1.0f / sqrtf(block_sum<256>(ss, red) / (float)dim + eps);
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int d = 4 * ((int)threadIdx.x + 256 * i);
            if (d < dim)
                store4(yrow + d, float4{wv[i].x * (ov[i].x * r) * sigmoid_f(gv[i].x), wv[i].y * (ov[i].y * r) * sigmoid_f(gv[i].y),
                                        wv[i].z * (ov[i].z * r) * sigmoid_f(gv[i].z), wv[i].w * (ov[i].w * r) * sigmoid_f(gv[i].w)});
        }
    } else {
        float ss = 0.f;
        for (int d = threadIdx.x; d < dim; d += 256) ss = fmaf(orow[d], orow[d], ss);
        const float r = 1.0f / sqrtf(block_sum<256>(ss, red) / (float)dim + eps);
        for (int d = threadIdx.x; d < dim; d += 256) store_f32(yrow, d, load_f32(w, d) * (orow[d] * r) * sigmoid_f(grow[d]));
    }
}

}  // namespace

GI_API int gi_lightning_max_key_dim() { return 512; }
GI_API int gi_lightning_chunk_rows() { return CHUNK; }

// proj: float32 [n_rows, ld], whose columns q_off.., k_off.. hold q and k [heads*dk] and v_off.. v [heads*dv], before SiLU; powers: float32
// [heads][65]; state: [slots, state_stride]; out: float32 [n_rows, ldo] gets the heads' results [heads*dv].  n_chunks 0: token by token;
// otherwise the step's rows in chunks (n_chunks of them: the sum over the requests of their rows over 64, rounded up), with `states` room
// for n_chunks * heads * dk * dv floats.
GI_API int gi_lightning_scan(const float* proj, long ld, int q_off, int k_off, int v_off, const float* powers, const int* seg_start, const int* seg_len, int n_segs,
                             const int* row_slot, float* state, long state_stride, float* out, long ldo, int n_heads, int dk, int dv, int n_chunks,
                             float* states, hipStream_t stream) {
    GI_REQUIRE(n_segs > 0 && n_heads > 0 && dk > 0 && dk <= 512 && dv > 0, "lightning_scan: bad sizes (runs %d, heads %d, dk %d, dv %d; dk at most 512)", n_segs, n_heads, dk, dv);
    GI_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && ld >= q_off + (long)n_heads * dk && ld >= k_off + (long)n_heads * dk && ld >= v_off + (long)n_heads * dv,
               "lightning_scan: the columns named lie outside the rows");
    GI_REQUIRE(state_stride >= (long)n_heads * dk * dv && ldo >= (long)n_heads * dv, "lightning_scan: state or output stride too small");
    const long per_head = (long)dk * dv;
    const int col_groups = (dv + SCAN_COLS - 1) / SCAN_COLS;
    GI_REQUIRE(n_heads <= 65535 && (per_head + 255) / 256 <= 65535 && col_groups <= 65535, "lightning_scan: too many heads or channels");
    if (n_chunks == 0) {
        dim3 grid(n_segs, n_heads, col_groups);
#define GO(R) lightning_scan_kernel<R><<<grid, 256, 0, stream>>>(proj, ld, q_off, k_off, v_off, powers, seg_start, seg_len, row_slot, state, state_stride, out, ldo, dk, dv)
        if (dk <= 32) GO(2); else if (dk <= 64) GO(4); else if (dk <= 128) GO(8); else if (dk <= 256) GO(16); else GO(32);
#undef GO
        GI_CHECK_LAUNCH("lightning_scan");
        return 0;
    }
    GI_REQUIRE(n_chunks > 0 && states != nullptr, "lightning_scan: rows in chunks need the chunks' scratch memory");
    const int tiles = ((dk + 31) / 32) * ((dv + 31) / 32);
    lightning_chunk_states_kernel<<<dim3(n_chunks, n_heads, (tiles + 3) / 4), 256, 0, stream>>>(proj, ld, k_off, v_off, powers, seg_start, seg_len, n_segs, states,
                                                                                               n_heads, dk, dv);
    GI_CHECK_LAUNCH("lightning_scan (chunks)");
    lightning_carry_kernel<<<dim3(n_segs, n_heads, (unsigned)((per_head + 255) / 256)), 256, 0, stream>>>(powers, seg_start, seg_len, row_slot, state, state_stride, states,
                                                                                                         n_heads, (int)per_head);
    GI_CHECK_LAUNCH("lightning_scan (carry)");
    lightning_chunk_rows_kernel<<<dim3(n_chunks, n_heads, (dv + 63) / 64), 256, 0, stream>>>(proj, ld, q_off, k_off, v_off, powers, seg_start, seg_len, n_segs, states,
                                                                                           out, ldo, n_heads, dk, dv);
    GI_CHECK_LAUNCH("lightning_scan (rows)");
    return 0;
}

GI_API int gi_row_norm_gate(const float* o, long ldo, const float* g, long ldg, const void* w, int w_dtype, void* y, int y_dtype, long ldy, int n_rows, int dim, float eps,
                            hipStream_t stream) {
    GI_REQUIRE(n_rows > 0 && dim > 0 && ldo >= dim && ldg >= dim && ldy >= dim, "row_norm_gate: bad sizes (rows %d, columns %d)", n_rows, dim);
    const bool fast = dim % 4 == 0 && dim <= 8192 && ldo % 4 == 0 && ldg % 4 == 0 && ldy % 4 == 0 && (((uintptr_t)o | (uintptr_t)g | (uintptr_t)w | (uintptr_t)y) & 15) == 0;
    const int nv = (dim + 1023) / 1024;
#define GO(NV, TW, TO) row_norm_gate_kernel<NV, TW, TO><<<n_rows, 256, 0, stream>>>(o, ldo, g, ldg, (const TW*)w, (TO*)y, ldy, dim, eps)
#define LAUNCH(TW, TO)                         \
    do {                                       \
        if (!fast) GO(0, TW, TO);              \
        else if (nv <= 1) GO(1, TW, TO);       \
        else if (nv <= 2) GO(2, TW, TO);       \
        else if (nv <= 4) GO(4, TW, TO);       \
        else GO(8, TW, TO);                    \
    } while (0)
    if (w_dtype == GI_F32 && y_dtype == GI_F32) LAUNCH(float, float);
    else if (w_dtype == GI_F32 && y_dtype == GI_BF16) LAUNCH(float, bf16_t);
    else if (w_dtype == GI_BF16 && y_dtype == GI_BF16) LAUNCH(bf16_t, bf16_t);
    else if (w_dtype == GI_BF16 && y_dtype == GI_F32) LAUNCH(bf16_t, float);
    else return gi_fail("row_norm_gate: unknown dtypes %d, %d", w_dtype, y_dtype);
#undef LAUNCH
#undef GO
    GI_CHECK_LAUNCH("row_norm_gate");
    return 0;
}
