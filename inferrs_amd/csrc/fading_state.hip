// A matrix a head whose ROWS fade, each by a factor of its own a token, and take in what the factor leaves open:
//     k_t = (1 - l) * sigmoid(-(z_t + b)),   f_t = 1 - k_t = l + (1 - l) * sigmoid(z_t + b)      (a gate a channel, l its floor)
//     S_t = diag(f_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T silu(u_t)                                S: [dim x vdim]
// and behind it an RMS norm a head with one weight of vdim entries (the HGRN2 recurrence; Qin et al., "HGRN2: Gated Linear
// RNNs with State Expansion").  u, z and v are slices of the projections' rows; everything between their load and the
// store of the normed output is 32-bit, the state included.
//
// What a request carries lies in its row of a 32-bit state array [slots][row_floats], the matrices as [head][column j of S,
// vdim][dim].  A new request's row is zero.  f_t is formed as 1 - k_t everywhere (the rows stay within the values' range,
// so an error of 2^-25 of f weighs no more than a rounding of S).
//
// Two forms.  fading_walk_kernel walks a request's tokens in order (decode steps, short portions).  Long portions are cut
// into chunks of 64 tokens that run side by side, in three kernels of matrix products in true 32-bit
// (v_mfma_f32_16x16x4_f32), for keys of up to 128 and values of up to 256 entries:
//   fading_local     a chunk's own matrix U = sum_s (prod_(r>s) f_r) k_s v_s^T and the products A of its factors;
//   fading_chunks    a request's chunks in order, S <- A S + U from the state row; the workspace keeps what each starts from;
//   fading_outputs   o_t = (prod_(r<=t) f_r q_t) S_c + sum_(s<=t) P[t][s] v_s and the norm behind it.
// The scores P[t][s] = sum_i q_t[i] k_s[i] prod_(s<r<=t) f_r[i] are no product of two matrices, and their factors cannot be
// split at one point of a chunk (a quotient of products would over- or underflow).  A chunk is cut into four blocks of 16
// tokens: between blocks the factor splits at the borders, q_t (prod from its block's start) . (whole blocks between) .
// k_s (prod to its block's end), every piece a product of numbers up to 1.  Inside a block the same once more between its four
// groups of 4 tokens (three products of the whole block, one a distance between groups, of which the pairs of groups at that
// distance are kept); inside a group the vector units form the ten scores directly.
#include "api.h"
#include "common.h"

#define FS_R 8
#define FS_THREADS 256
#define FS_CHUNK 64
#define FS_SUB 16
#define FS_V_LD 36
#define FS_MAX_DIM 128
#define FS_MAX_VDIM 256

typedef float fs_f32x4 __attribute__((ext_vector_type(4)));

struct FadingArgs {
    void* out;                        // [n][H * vdim], normed (chunks), or 32-bit as it is (walk)
    float* state; long long row_floats, s_off;
    const void* proj; long long ld; int q_off, f_off, v_off;
    const float *f_bias, *lower;      // [H * dim]
    const float* norm_w; float eps;   // [vdim]
    const int *cu_tokens, *state_slots;
    int H, dim, vdim, cols, stage, wide, vec;
    int chunk0, chunks;               // chunks of this pass: the first one's number in its request, how many a request
    float *chunk_s, *chunk_a;         // [seqs][chunks][H][vdim][dim], [seqs][chunks][H][dim]
};

__device__ __forceinline__ float fs_open(float z, float b, float l) { return (1.0f - l) / (1.0f + expf(z + b)); }
__device__ __forceinline__ float fs_silu(float u) { return u / (1.0f + expf(-u)); }

// ---- token by token ---------------------------------------------------------------------------------------------------
// A block owns a (request, head, tile of S's columns); a column is shared by P neighbouring lanes, each with FS_R of its
// entries in registers; the operands of a stage of tokens come into shared memory together.
template <typename T, int P>
__global__ __launch_bounds__(FS_THREADS) void fading_walk_kernel(const FadingArgs a) {
    extern __shared__ __attribute__((aligned(16))) float fs_stage[];
    constexpr int dimp = P * FS_R;
    float* const q_s = fs_stage;
    float* const k_s = q_s + (size_t)a.stage * dimp;
    float* const v_s = k_s + (size_t)a.stage * dimp;
    const int p = threadIdx.x % P, jj = threadIdx.x / P;
    const int h = blockIdx.y, seq = blockIdx.z;
    const int j0 = blockIdx.x * a.cols, j = j0 + jj;
    const bool live = j < a.vdim;
    const int first = a.cu_tokens[seq], last = a.cu_tokens[seq + 1];
    const int i0 = p * FS_R;
    const T* q = (const T*)a.proj + a.q_off + (long long)h * a.dim;
    const T* z = (const T*)a.proj + a.f_off + (long long)h * a.dim;
    const T* v = (const T*)a.proj + a.v_off + (long long)h * a.vdim;
    float* srow = a.state + (long long)a.state_slots[seq] * a.row_floats + a.s_off + ((long long)h * a.vdim + (live ? j : 0)) * a.dim + i0;
    const bool wide = a.wide && i0 + FS_R <= a.dim;
    float S[FS_R];
    if (live && wide) {
        const float4 lo = *(const float4*)srow, hi = *(const float4*)(srow + 4);
        S[0] = lo.x; S[1] = lo.y; S[2] = lo.z; S[3] = lo.w; S[4] = hi.x; S[5] = hi.y; S[6] = hi.z; S[7] = hi.w;
    } else {
#pragma unroll
        for (int r = 0; r < FS_R; ++r) S[r] = (live && i0 + r < a.dim) ? srow[r] : 0.f;
    }
    for (int t0 = first; t0 < last; t0 += a.stage) {
        const int nt = last - t0 < a.stage ? last - t0 : a.stage;
        __syncthreads();                                          // (the stage before is used up)
        for (int e = threadIdx.x; e < nt * dimp; e += FS_THREADS) {
            const int tt = e / dimp, i = e - tt * dimp;
            float qv = 0.f, kv = 0.f;
            if (i < a.dim) {
                qv = fs_silu(ld(q + (long long)(t0 + tt) * a.ld + i));
                kv = fs_open(ld(z + (long long)(t0 + tt) * a.ld + i), a.f_bias[h * a.dim + i], a.lower[h * a.dim + i]);
            }
            q_s[e] = qv;
            k_s[e] = kv;
        }
        for (int e = threadIdx.x; e < nt * a.cols; e += FS_THREADS) {
            const int tt = e / a.cols, jv = j0 + e - tt * a.cols;
            v_s[e] = jv < a.vdim ? ld(v + (long long)(t0 + tt) * a.ld + jv) : 0.f;
        }
        __syncthreads();
#pragma unroll 2
        for (int tt = 0; tt < nt; ++tt) {
            const float4 qa = *(const float4*)(q_s + tt * dimp + i0), qb = *(const float4*)(q_s + tt * dimp + i0 + 4);
            const float4 ka = *(const float4*)(k_s + tt * dimp + i0), kb = *(const float4*)(k_s + tt * dimp + i0 + 4);
            const float qc[FS_R] = {qa.x, qa.y, qa.z, qa.w, qb.x, qb.y, qb.z, qb.w};
            const float kc[FS_R] = {ka.x, ka.y, ka.z, ka.w, kb.x, kb.y, kb.z, kb.w};
            const float vc = v_s[tt * a.cols + jj];
            float part = 0.f;
#pragma unroll
            for (int r = 0; r < FS_R; ++r) {
                S[r] = fmaf(1.0f - kc[r], S[r], kc[r] * vc);
                part = fmaf(S[r], qc[r], part);
            }
#pragma unroll
            for (int o = P / 2; o > 0; o >>= 1) part += __shfl_xor(part, o, IA_WAVE);
            if (p == 0 && live) ((float*)a.out)[((long long)(t0 + tt) * a.H + h) * a.vdim + j] = part;
        }
    }
    if (live && wide) {
        *(float4*)srow = make_float4(S[0], S[1], S[2], S[3]);
        *(float4*)(srow + 4) = make_float4(S[4], S[5], S[6], S[7]);
    } else if (live) {
#pragma unroll
        for (int r = 0; r < FS_R; ++r)
            if (i0 + r < a.dim) srow[r] = S[r];
    }
}

// ---- chunks side by side ----------------------------------------------------------------------------------------------
// The kernels below are compiled for keys of up to 16 KT entries (KT 2, 4 or 8; what lies between dim and 16 KT is zeros in
// shared memory): with every count and every pitch a constant a wave's operand reads and products stand in one piece, where
// tests between them left each product waiting for its own reads (a chunk's outputs 42 us alone on a compute unit).
//
// Rows of a chunk into shared memory: dst[tt][i] = fn(src[(first + tt) * ld + i], c[i]) for tt < nt, i < dim, zeros up to 64
// rows and 16 KT columns.  A thread owns one 16-byte piece of a row (with `vec`; else one column) of several rows: what fn
// needs of its columns (`consts(i)`) is read once, and every load is asked for before the first is used.
__device__ __forceinline__ void fs_load(const float* p, float (&v)[8]) {
    const float4 q = *(const float4*)p;
    v[0] = q.x; v[1] = q.y; v[2] = q.z; v[3] = q.w;
}
__device__ __forceinline__ void fs_load(const bf16_t* p, float (&v)[8]) {
    const uint4 q = *(const uint4*)p;
    const uint32_t w[4] = {q.x, q.y, q.z, q.w};
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        v[2 * e] = __uint_as_float(w[e] << 16);
        v[2 * e + 1] = __uint_as_float(w[e] & 0xffff0000u);
    }
}

template <typename T, int KT, typename C, typename F>
__device__ __forceinline__ void fs_stage_rows(float* __restrict__ dst, const T* __restrict__ src, long long ld_g, int first, int nt,
                                              int dim, bool vec, C consts, F fn) {
    constexpr int D16 = 16 * KT, LD = D16 + 4, E = 16 / (int)sizeof(T);
    if (vec) {                                             // (dim is a multiple of E, the rows start at multiples of 16 bytes)
        constexpr int PPR = D16 / E, STEP = FS_THREADS / PPR, ITERS = FS_CHUNK / STEP;
        const int piece = threadIdx.x % PPR, row0 = threadIdx.x / PPR;
        const bool inside = piece * E < dim;
        float v[ITERS][8];
#pragma unroll
        for (int it = 0; it < ITERS; ++it) {
            const int tt = row0 + it * STEP;
            fs_load(src + (long long)(first + (tt < nt ? tt : nt - 1)) * ld_g + (inside ? piece * E : 0), v[it]);
        }
        float2 c[E];
#pragma unroll
        for (int e = 0; e < E; ++e) c[e] = consts(inside ? piece * E + e : 0);
#pragma unroll
        for (int it = 0; it < ITERS; ++it) {
            const int tt = row0 + it * STEP;
            const bool live = inside && tt < nt;
#pragma unroll
            for (int e = 0; e < E; e += 4) {
                float w[4];
#pragma unroll
                for (int x = 0; x < 4; ++x) w[x] = live ? fn(v[it][e + x], c[e + x]) : 0.f;
                *(float4*)(dst + tt * LD + piece * E + e) = make_float4(w[0], w[1], w[2], w[3]);
            }
        }
        return;
    }
    constexpr int STEP = FS_THREADS / D16;
    const int i = threadIdx.x % D16;
    const float2 c = consts(i < dim ? i : 0);
#pragma unroll 8
    for (int tt = threadIdx.x / D16; tt < FS_CHUNK; tt += STEP)
        dst[tt * LD + i] = tt < nt && i < dim ? fn(ld(src + (long long)(first + tt) * ld_g + i), c) : 0.f;
}

// 32 columns of v, v_s[tt][c] (zeros for tokens the chunk does not have and columns beyond vdim): into registers, and from
// there into shared memory.
template <typename T>
__device__ __forceinline__ void fs_fetch_values(float (&vv)[8], const T* __restrict__ v, long long ld_g, int first, int nt, int j0, int vdim) {
    const int j = j0 + (threadIdx.x & 31);
#pragma unroll
    for (int it = 0; it < 8; ++it) {
        const int tt = (threadIdx.x >> 5) + 8 * it;
        vv[it] = tt < nt && j < vdim ? ld(v + (long long)(first + tt) * ld_g + j) : 0.f;
    }
}
__device__ __forceinline__ void fs_put_values(float* __restrict__ v_s, const float (&vv)[8]) {
#pragma unroll
    for (int it = 0; it < 8; ++it) v_s[((threadIdx.x >> 5) + 8 * it) * FS_V_LD + (threadIdx.x & 31)] = vv[it];
}

// A block of four waves owns a (chunk, head).
template <typename T, int KT>
__global__ __launch_bounds__(FS_THREADS) void fading_local_kernel(const FadingArgs a) {
    extern __shared__ __attribute__((aligned(16))) float fs_shared[];
    constexpr int D16 = 16 * KT, LD = D16 + 4, MT = (KT + 3) / 4;
    float* const k_s = fs_shared;                          // [64][LD]
    float* const v_s = k_s + FS_CHUNK * LD;                // [64][FS_V_LD]
    float* const m_s = v_s + FS_CHUNK * FS_V_LD;           // [4][D16]: the products of the blocks' factors
    const int h = blockIdx.y;
    const int seq = blockIdx.z / a.chunks, c = blockIdx.z - seq * a.chunks;
    const int first = a.cu_tokens[seq] + (a.chunk0 + c) * FS_CHUNK, end = a.cu_tokens[seq + 1];
    if (first >= end) return;                              // (the whole block: this request has fewer chunks)
    const int nt = end - first < FS_CHUNK ? end - first : FS_CHUNK;
    const float *fb = a.f_bias + h * a.dim, *lo = a.lower + h * a.dim;
    const T* v = (const T*)a.proj + a.v_off + (long long)h * a.vdim;
    float vv[8];                                           // (columns of v are on their way while those before are multiplied)
    fs_fetch_values<T>(vv, v, a.ld, first, nt, 0, a.vdim);
    fs_stage_rows<T, KT>(k_s, (const T*)a.proj + a.f_off + (long long)h * a.dim, a.ld, first, nt, a.dim, a.vec != 0,
                         [&](int i) { return make_float2(fb[i], lo[i]); }, [](float z, float2 g) { return fs_open(z, g.x, g.y); });
    __syncthreads();
    // (tokens the chunk does not have are zeros: their factor is 1)
#pragma unroll
    for (int e = threadIdx.x; e < 4 * D16; e += FS_THREADS) {
        const int sub = e / D16, i = e - sub * D16;
        float kk[FS_SUB], run = 1.f;
#pragma unroll
        for (int s = 0; s < FS_SUB; ++s) kk[s] = k_s[(FS_SUB * sub + s) * LD + i];
#pragma unroll
        for (int s = FS_SUB - 1; s >= 0; --s) {
            k_s[(FS_SUB * sub + s) * LD + i] = kk[s] * run;
            run *= 1.0f - kk[s];
        }
        m_s[e] = run;
    }
    __syncthreads();
    const long long unit = (long long)blockIdx.z * a.H + h;
    for (int i = threadIdx.x; i < a.dim; i += FS_THREADS)
        a.chunk_a[unit * a.dim + i] = m_s[i] * m_s[D16 + i] * m_s[2 * D16 + i] * m_s[3 * D16 + i];
    float* const u_out = a.chunk_s + unit * a.vdim * a.dim;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int r16 = lane & 15, kq = lane >> 4;
    // the wave's rows of U: tiles wave, wave + 4; their keys, to the chunk's end, stay in registers
    float ak[MT][FS_CHUNK / 4];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        const int mt = wave + 4 * m, ii = 16 * (mt < KT ? mt : 0) + r16;
        const float m1 = m_s[D16 + ii], m2 = m_s[2 * D16 + ii], m3 = m_s[3 * D16 + ii];
        const float later[4] = {m1 * m2 * m3, m2 * m3, m3, 1.0f};
#pragma unroll
        for (int k4 = 0; k4 < FS_CHUNK / 4; ++k4) ak[m][k4] = k_s[(4 * k4 + kq) * LD + ii] * later[4 * k4 / FS_SUB];
    }
    for (int j0 = 0; j0 < a.vdim; j0 += 32) {
        if (j0 > 0) __syncthreads();                       // (the columns before are used up)
        fs_put_values(v_s, vv);
        if (j0 + 32 < a.vdim) fs_fetch_values<T>(vv, v, a.ld, first, nt, j0 + 32, a.vdim);
        __syncthreads();
        const float* vb = v_s + kq * FS_V_LD + r16;
        fs_f32x4 acc[MT][2];
#pragma unroll
        for (int m = 0; m < MT; ++m) acc[m][0] = acc[m][1] = (fs_f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k4 = 0; k4 < FS_CHUNK / 4; ++k4) {
            const float b0 = vb[4 * k4 * FS_V_LD], b1 = vb[4 * k4 * FS_V_LD + 16];
#pragma unroll
            for (int m = 0; m < MT; ++m) {
                acc[m][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(ak[m][k4], b0, acc[m][0], 0, 0, 0);
                acc[m][1] = __builtin_amdgcn_mfma_f32_16x16x4f32(ak[m][k4], b1, acc[m][1], 0, 0, 0);
            }
        }
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int c2 = 0; c2 < 2; ++c2) {
                const int col = j0 + 16 * c2 + r16, i = 16 * (wave + 4 * m) + 4 * kq;
                if (wave + 4 * m >= KT || col >= a.vdim) continue;
                float* at = u_out + (long long)col * a.dim + i;
                if (a.wide && i + 4 <= a.dim) *(float4*)at = make_float4(acc[m][c2][0], acc[m][c2][1], acc[m][c2][2], acc[m][c2][3]);
                else {
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        if (i + r < a.dim) at[r] = acc[m][c2][r];
                }
            }
    }
}

// A request's chunks in order, one thread an entry of the heads' matrices; eight chunks' entries are asked for at a time.
__global__ void fading_chunks_kernel(const FadingArgs a) {
    const long long e = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    const int per_head = a.vdim * a.dim;
    const long long per_seq = (long long)a.H * per_head;
    if (e >= per_seq) return;
    const int seq = blockIdx.y;
    const int h = (int)(e / per_head), i = (int)(e % a.dim);
    int n = (a.cu_tokens[seq + 1] - a.cu_tokens[seq] + FS_CHUNK - 1) / FS_CHUNK - a.chunk0;
    n = n < a.chunks ? n : a.chunks;
    if (n <= 0) return;
    float* srow = a.state + (long long)a.state_slots[seq] * a.row_floats + a.s_off + e;
    float S = *srow;
    for (int c0 = 0; c0 < n; c0 += 8) {
        float u[8], f[8];
#pragma unroll
        for (int q = 0; q < 8; ++q) {
            if (c0 + q >= n) continue;
            const long long unit = (long long)seq * a.chunks + c0 + q;
            u[q] = a.chunk_s[unit * per_seq + e];
            f[q] = a.chunk_a[(unit * a.H + h) * a.dim + i];
        }
#pragma unroll
        for (int q = 0; q < 8; ++q) {
            if (c0 + q >= n) continue;
            a.chunk_s[((long long)seq * a.chunks + c0 + q) * per_seq + e] = S;
            S = fmaf(f[q], S, u[q]);
        }
    }
    *srow = S;
}

// A block of four waves owns a (chunk, head); wave w owns tokens 16 w .. 16 w + 15.  Shared memory: the queries, whose
// rows the scores replace once a wave has its own in registers; the keys, whose place the columns of v and of the matrix
// the chunk starts from take once the scores are formed.  NT: pairs of 16-column tiles that a wave keeps in registers.
template <typename T, int KT, int NT>
__global__ __launch_bounds__(FS_THREADS, 2) void fading_outputs_kernel(const FadingArgs a) {
    extern __shared__ __attribute__((aligned(16))) float fs_shared[];
    constexpr int D16 = 16 * KT, LD = D16 + 4, P_LD = LD >= FS_CHUNK + 4 ? LD : FS_CHUNK + 4;
    constexpr int TILES = FS_CHUNK * FS_V_LD + 32 * LD, K_FLOATS = FS_CHUNK * LD > TILES ? FS_CHUNK * LD : TILES;
    float* const q_s = fs_shared;                          // [64][LD]
    float* const k_s = q_s + FS_CHUNK * P_LD;              // [64][LD]
    float* const m_s = k_s + K_FLOATS;                     // [4][D16]: the products of the blocks' factors
    float* const g_s = m_s + 4 * D16;                      // [4][4][D16]: of the groups of 4 tokens
    float* const p_s = q_s;                                // [64][P_LD], in the queries' rows (or rows of 68 where those are shorter)
    float* const v_s = k_s;                                // [64][FS_V_LD]
    float* const c_s = v_s + FS_CHUNK * FS_V_LD;           // [32][LD]
    const int h = blockIdx.y;
    const int seq = blockIdx.z / a.chunks, c = blockIdx.z - seq * a.chunks;
    const int first = a.cu_tokens[seq] + (a.chunk0 + c) * FS_CHUNK, end = a.cu_tokens[seq + 1];
    if (first >= end) return;                              // (the whole block)
    const int nt = end - first < FS_CHUNK ? end - first : FS_CHUNK;
    const float *fb = a.f_bias + h * a.dim, *lo = a.lower + h * a.dim;
    const T* v = (const T*)a.proj + a.v_off + (long long)h * a.vdim;
    fs_stage_rows<T, KT>(q_s, (const T*)a.proj + a.q_off + (long long)h * a.dim, a.ld, first, nt, a.dim, a.vec != 0,
                         [](int) { return make_float2(0.f, 0.f); }, [](float u, float2) { return fs_silu(u); });
    fs_stage_rows<T, KT>(k_s, (const T*)a.proj + a.f_off + (long long)h * a.dim, a.ld, first, nt, a.dim, a.vec != 0,
                         [&](int i) { return make_float2(fb[i], lo[i]); }, [](float z, float2 g) { return fs_open(z, g.x, g.y); });
    __syncthreads();
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int r16 = lane & 15, kq = lane >> 4;
    float* const q0 = q_s + FS_SUB * wave * LD;          // the wave's block of 16 tokens
    float* const k0 = k_s + FS_SUB * wave * LD;
    const int grp = r16 >> 2;                              // the group of 4 of row (or column) r16 of the block
    // ---- the scores inside the groups: lane (t, part) has token t and a quarter of the channels; a running product of the
    // factors stands with the query: near[e] is the score of token t - e (of the same group)
    float near[4] = {0.f, 0.f, 0.f, 0.f};
    {
#pragma unroll
        for (int j = 0; j < KT; ++j) {
            const float4 q4 = *(const float4*)(q0 + r16 * LD + 16 * j + 4 * kq);
            float qf[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int s = r16 - e > 4 * grp ? r16 - e : 4 * grp;     // (beyond the group's first token: not used)
                const float4 k4 = *(const float4*)(k0 + s * LD + 16 * j + 4 * kq);
                const float kk[4] = {k4.x, k4.y, k4.z, k4.w};
#pragma unroll
                for (int x = 0; x < 4; ++x) {
                    near[e] = fmaf(qf[x], kk[x], near[e]);
                    qf[x] *= 1.0f - kk[x];
                }
            }
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            near[e] += __shfl_xor(near[e], 16, IA_WAVE);
            near[e] += __shfl_xor(near[e], 32, IA_WAVE);
        }
    }
    __builtin_amdgcn_wave_barrier();
    asm volatile("" ::: "memory");
    // ---- the groups' own products: q_t from the group's start, k_s to its end (the wave's own rows: no barrier)
    float* const g_w = g_s + 4 * wave * D16;               // [4][D16]: the products of the groups' factors
    for (int i = lane; i < D16; i += IA_WAVE) {
        float kk[FS_SUB], qq[FS_SUB];
#pragma unroll
        for (int s = 0; s < FS_SUB; ++s) { kk[s] = k0[s * LD + i]; qq[s] = q0[s * LD + i]; }
#pragma unroll
        for (int a4 = 0; a4 < 4; ++a4) {
            float run = 1.f, back = 1.f;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                run *= 1.0f - kk[4 * a4 + e];
                q0[(4 * a4 + e) * LD + i] = qq[4 * a4 + e] * run;
            }
            g_w[a4 * D16 + i] = run;
#pragma unroll
            for (int e = 3; e >= 0; --e) {
                k0[(4 * a4 + e) * LD + i] = kk[4 * a4 + e] * back;
                back *= 1.0f - kk[4 * a4 + e];
            }
        }
    }
    __builtin_amdgcn_wave_barrier();
    asm volatile("" ::: "memory");
    // ---- between the groups of the block: row t of the queries goes back one whole group a pass, until it stands at the
    // block's start
    float aq[4 * KT];
#pragma unroll
    for (int kk = 0; kk < 4 * KT; ++kk) aq[kk] = q0[r16 * LD + 4 * kk + kq];
    float inside[4] = {0.f, 0.f, 0.f, 0.f};                // rows 4 kq + r, column r16
#pragma unroll
    for (int back = 1; back < 4; ++back) {
        fs_f32x4 acc = (fs_f32x4){0.f, 0.f, 0.f, 0.f};
        const float* kb = k0 + r16 * LD + kq;
#pragma unroll
        for (int kk = 0; kk < 4 * KT; ++kk)
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(aq[kk], kb[4 * kk], acc, 0, 0, 0);
        const bool mine = kq - grp == back;                // (rows 4 kq + r are group kq, column r16 is group grp)
#pragma unroll
        for (int r = 0; r < 4; ++r) inside[r] = mine ? acc[r] : inside[r];
        const float* gb = g_w + (grp >= back ? grp - back : 0) * D16 + kq;
#pragma unroll
        for (int kk = 0; kk < 4 * KT; ++kk)
            aq[kk] *= grp >= back ? gb[4 * kk] : 1.0f;
    }
    __builtin_amdgcn_wave_barrier();
    asm volatile("" ::: "memory");
    // ---- the keys to the block's end
    for (int i = lane; i < D16; i += IA_WAVE) {
        const float m1 = g_w[D16 + i], m2 = g_w[2 * D16 + i], m3 = g_w[3 * D16 + i];
        const float later[3] = {m1 * m2 * m3, m2 * m3, m3};
#pragma unroll
        for (int s = 0; s < 12; ++s) k0[s * LD + i] *= later[s / 4];
        m_s[wave * D16 + i] = g_w[i] * later[0];
    }
    __syncthreads();                                       // (the other waves' keys and products; and their queries, which are read)
    float* const mine = p_s + FS_SUB * wave * P_LD;
#pragma unroll
    for (int r = 0; r < 4; ++r) mine[(4 * kq + r) * P_LD + FS_SUB * wave + r16] = inside[r];
    __builtin_amdgcn_wave_barrier();
    asm volatile("" ::: "memory");
#pragma unroll
    for (int e = 0; e < 4; ++e)
        if (kq == e && r16 - e >= 4 * grp) mine[r16 * P_LD + FS_SUB * wave + r16 - e] = near[e];
    for (int cb = wave - 1; cb >= 0; --cb) {
        fs_f32x4 acc = (fs_f32x4){0.f, 0.f, 0.f, 0.f};
        const float* kb = k_s + (FS_SUB * cb + r16) * LD + kq;
#pragma unroll
        for (int kk = 0; kk < 4 * KT; ++kk)
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(aq[kk], kb[4 * kk], acc, 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) mine[(4 * kq + r) * P_LD + FS_SUB * cb + r16] = acc[r];
#pragma unroll
        for (int kk = 0; kk < 4 * KT; ++kk)
            aq[kk] *= m_s[cb * D16 + 4 * kk + kq];
    }
    // ---- the outputs, 32 columns at a time; the next columns of v and of the matrix the chunk starts from are on their way
    // in registers while these are multiplied
    const float* start = a.chunk_s + ((long long)blockIdx.z * a.H + h) * a.vdim * a.dim;
    constexpr int per_row = D16 / 4;                       // 16-byte pieces of a column of the matrix
    float vv[8];
    float4 cc[KT / 2];
    auto fetch = [&](int j0) {
        fs_fetch_values<T>(vv, v, a.ld, first, nt, j0, a.vdim);
        if (!a.wide) return;
#pragma unroll
        for (int it = 0; it < KT / 2; ++it) {
            const int idx = threadIdx.x + it * FS_THREADS, jj = idx / per_row, piece = idx - jj * per_row;
            cc[it] = jj < 32 && j0 + jj < a.vdim && 4 * piece < a.dim ? *(const float4*)(start + (long long)(j0 + jj) * a.dim + 4 * piece)
                                                                      : make_float4(0.f, 0.f, 0.f, 0.f);
        }
    };
    fetch(0);
    float nw[NT][2];                                       // the norm's weights of the lane's columns
#pragma unroll
    for (int jt = 0; jt < NT; ++jt)
#pragma unroll
        for (int c2 = 0; c2 < 2; ++c2) nw[jt][c2] = a.norm_w[32 * jt + 16 * c2 + r16 < a.vdim ? 32 * jt + 16 * c2 + r16 : 0];
    fs_f32x4 acc[NT][2];
#pragma unroll
    for (int jt = 0; jt < NT; ++jt) {
        acc[jt][0] = acc[jt][1] = (fs_f32x4){0.f, 0.f, 0.f, 0.f};
        const int j0 = 32 * jt;
        if (j0 >= a.vdim) continue;
        __syncthreads();                                   // (the keys, or the columns before, are used up)
        fs_put_values(v_s, vv);
        if (a.wide) {
#pragma unroll
            for (int it = 0; it < KT / 2; ++it) {
                const int idx = threadIdx.x + it * FS_THREADS, jj = idx / per_row, piece = idx - jj * per_row;
                if (jj < 32) *(float4*)(c_s + jj * LD + 4 * piece) = cc[it];
            }
        } else {
            for (int e = threadIdx.x; e < 32 * D16; e += FS_THREADS) {
                const int jj = e / D16, i = e - jj * D16;
                c_s[jj * LD + i] = (j0 + jj < a.vdim && i < a.dim) ? start[(long long)(j0 + jj) * a.dim + i] : 0.f;
            }
        }
        if (j0 + 32 < a.vdim) fetch(j0 + 32);
        __syncthreads();
        const float* sb = c_s + r16 * LD + kq;
#pragma unroll
        for (int kk = 0; kk < 4 * KT; ++kk) {
            acc[jt][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(aq[kk], sb[4 * kk], acc[jt][0], 0, 0, 0);
            acc[jt][1] = __builtin_amdgcn_mfma_f32_16x16x4f32(aq[kk], sb[16 * LD + 4 * kk], acc[jt][1], 0, 0, 0);
        }
        const float* pa = mine + r16 * P_LD + kq;
        const float* vb = v_s + kq * FS_V_LD + r16;
        for (int kb = 0; kb <= wave; ++kb) {
#pragma unroll
            for (int k0 = 0; k0 < FS_SUB; k0 += 4) {
                const float av = pa[FS_SUB * kb + k0];
                const float* vk = vb + (FS_SUB * kb + k0) * FS_V_LD;
                acc[jt][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(av, vk[0], acc[jt][0], 0, 0, 0);
                acc[jt][1] = __builtin_amdgcn_mfma_f32_16x16x4f32(av, vk[16], acc[jt][1], 0, 0, 0);
            }
        }
    }
    // ---- the norm over a head's columns, row by row (the 16 lanes of a row's values hold its columns)
    float rs[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int jt = 0; jt < NT; ++jt)
#pragma unroll
        for (int c2 = 0; c2 < 2; ++c2)
#pragma unroll
            for (int r = 0; r < 4; ++r) rs[r] = fmaf(acc[jt][c2][r], acc[jt][c2][r], rs[r]);   // (columns beyond vdim are zero)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
#pragma unroll
        for (int o = 8; o > 0; o >>= 1) rs[r] += __shfl_xor(rs[r], o, IA_WAVE);
        rs[r] = 1.0f / sqrtf(rs[r] / (float)a.vdim + a.eps);
    }
#pragma unroll
    for (int jt = 0; jt < NT; ++jt)
#pragma unroll
        for (int c2 = 0; c2 < 2; ++c2) {
            const int col = 32 * jt + 16 * c2 + r16;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int tt = FS_SUB * wave + 4 * kq + r;
                if (tt < nt && col < a.vdim) st((T*)a.out + ((long long)(first + tt) * a.H + h) * a.vdim + col, acc[jt][c2][r] * rs[r] * nw[jt][c2]);
            }
        }
}

// Floats of workspace for passes of `chunks` chunks a request.
extern "C" long long ia_fading_scan_workspace(int n_seqs, int chunks, int H, int dim, int vdim) {
    return (long long)n_seqs * chunks * ((long long)H * vdim * dim + (long long)H * dim);
}

static int fading_shared(const void* fn, int bytes, int& asked, const char* who) {
    if (bytes > asked && bytes > 64 * 1024) {
        const hipError_t e = hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);
        IA_CHECK(e == hipSuccess, "%s: cannot ask for %d bytes of shared memory: %s", who, bytes, hipGetErrorString(e));
        asked = 96 * 1024;
    }
    IA_CHECK(bytes <= 96 * 1024, "%s: %d bytes of shared memory", who, bytes);
    return 0;
}

// chunks 0: every request's tokens are walked from its state row; out is 32-bit and not normed.  chunks > 0: chunks of 64
// tokens side by side, `chunks` of a request at a time (max_q_len: the most tokens a request brings); out is normed, in the
// precision of proj.  q, the gate's logits and v lie at q_off, f_off and v_off of proj's rows.
extern "C" int ia_fading_scan(void* out, float* state, long long row_floats, long long s_off, const void* proj, long long ld, int q_off,
                              int f_off, int v_off, const float* f_bias, const float* lower, const float* norm_w, float eps,
                              const int* cu_tokens, const int* state_slots, int n_seqs, int H, int dim, int vdim, int max_q_len,
                              int chunks, float* workspace, int dtype, hipStream_t stream) {
    IA_CHECK(n_seqs >= 0 && H > 0 && dim > 0 && vdim > 0 && max_q_len >= 1, "fading_scan: bad sizes heads=%d dim=%d vdim=%d", H, dim, vdim);
    IA_CHECK(dim <= FS_R * IA_WAVE, "fading_scan: a key size of %d is beyond %d", dim, FS_R * IA_WAVE);
    IA_CHECK(s_off >= 0 && s_off + (long long)H * vdim * dim <= row_floats, "fading_scan: the matrices do not fit the state row");
    IA_CHECK(q_off >= 0 && q_off + (long long)H * dim <= ld && f_off >= 0 && f_off + (long long)H * dim <= ld && v_off >= 0 &&
             v_off + (long long)H * vdim <= ld, "fading_scan: q, f or v lie outside their rows");
    IA_CHECK(dtype == IA_F32 || dtype == IA_BF16, "fading_scan: unknown dtype %d", dtype);
    if (n_seqs == 0) return 0;
    FadingArgs a;
    a.out = out; a.state = state; a.row_floats = row_floats; a.s_off = s_off;
    a.proj = proj; a.ld = ld; a.q_off = q_off; a.f_off = f_off; a.v_off = v_off;
    a.f_bias = f_bias; a.lower = lower; a.norm_w = norm_w; a.eps = eps; a.cu_tokens = cu_tokens; a.state_slots = state_slots;
    a.H = H; a.dim = dim; a.vdim = vdim; a.cols = 0; a.stage = 0; a.chunk0 = 0; a.chunks = 0; a.chunk_s = a.chunk_a = nullptr;
    a.wide = dim % 4 == 0 && s_off % 4 == 0 && row_floats % 4 == 0 && (((uintptr_t)state | (uintptr_t)workspace) & 15) == 0;
    const int per = dtype == IA_F32 ? 4 : 8;
    a.vec = dim % per == 0 && q_off % per == 0 && f_off % per == 0 && ld % per == 0 && ((uintptr_t)proj & 15) == 0;
    if (chunks == 0) {
        int P = 1;
        while (P * FS_R < dim) P *= 2;
        a.cols = FS_THREADS / P;
        const int per_token = 2 * P * FS_R + a.cols;
        int stage = 32 * 1024 / 4 / per_token;
        stage = stage > 32 ? 32 : stage < 2 ? 2 : stage;
        a.stage = stage < max_q_len ? stage : max_q_len;
        const size_t shm = (size_t)a.stage * per_token * sizeof(float);
        const dim3 grid((unsigned)((vdim + a.cols - 1) / a.cols), (unsigned)H, (unsigned)n_seqs);
        IA_CHECK(H <= 65535 && n_seqs <= 65535, "fading_scan: %d heads of %d requests exceed the grid", H, n_seqs);
#define FS_WALK(PP)                                                                                         \
    do {                                                                                                    \
        if (dtype == IA_F32) fading_walk_kernel<float, PP><<<grid, FS_THREADS, shm, stream>>>(a);           \
        else fading_walk_kernel<bf16_t, PP><<<grid, FS_THREADS, shm, stream>>>(a);                          \
    } while (0)
        switch (P) {
            case 1: FS_WALK(1); break;
            case 2: FS_WALK(2); break;
            case 4: FS_WALK(4); break;
            case 8: FS_WALK(8); break;
            case 16: FS_WALK(16); break;
            case 32: FS_WALK(32); break;
            default: FS_WALK(64); break;
        }
#undef FS_WALK
        IA_LAUNCH_CHECK("fading_scan");
        return 0;
    }
    IA_CHECK(dim <= FS_MAX_DIM && vdim <= FS_MAX_VDIM && workspace != nullptr && norm_w != nullptr && chunks > 0,
             "fading_scan: chunks take keys up to %d, values up to %d, a workspace and the norm's weight", FS_MAX_DIM, FS_MAX_VDIM);
    IA_CHECK((long long)n_seqs * chunks <= 65535 && H <= 65535, "fading_scan: %d requests x %d chunks exceed the grid", n_seqs, chunks);
    a.chunks = chunks;
    a.chunk_s = workspace;
    a.chunk_a = workspace + (long long)n_seqs * chunks * H * vdim * dim;
    const dim3 cgrid(1, (unsigned)H, (unsigned)(n_seqs * chunks));
    const dim3 sgrid((unsigned)(((long long)H * vdim * dim + 255) / 256), (unsigned)n_seqs);
    static int asked[2][3][2];
    for (a.chunk0 = 0; (long long)a.chunk0 * FS_CHUNK < max_q_len; a.chunk0 += chunks) {
#define FS_LOCAL(TT, KT)                                                                                                  \
    fading_local_kernel<TT, KT><<<cgrid, FS_THREADS, (FS_CHUNK * (16 * KT + 4 + FS_V_LD) + 4 * 16 * KT) * 4, stream>>>(a)
#define FS_OUT(TT, KT, NT, I, J, K)                                                                                       \
    do {                                                                                                                  \
        constexpr int ld_s = 16 * KT + 4, p_ld = ld_s >= FS_CHUNK + 4 ? ld_s : FS_CHUNK + 4;                             \
        constexpr int tiles = FS_CHUNK * FS_V_LD + 32 * ld_s, k_floats = FS_CHUNK * ld_s > tiles ? FS_CHUNK * ld_s : tiles; \
        constexpr int oshm = (FS_CHUNK * p_ld + k_floats + 20 * 16 * KT) * 4;                                             \
        if (fading_shared((const void*)fading_outputs_kernel<TT, KT, NT>, oshm, asked[I][J][K], "fading_scan")) return 1;    \
        fading_outputs_kernel<TT, KT, NT><<<cgrid, FS_THREADS, oshm, stream>>>(a);                                        \
    } while (0)
#define FS_BOTH(TT, I)                                                                                                    \
    do {                                                                                                                  \
        if (dim <= 32) FS_LOCAL(TT, 2); else if (dim <= 64) FS_LOCAL(TT, 4); else FS_LOCAL(TT, 8);                         \
        fading_chunks_kernel<<<sgrid, 256, 0, stream>>>(a);                                                               \
        if (vdim <= 128) {                                                                                                \
            if (dim <= 32) FS_OUT(TT, 2, 4, I, 0, 0); else if (dim <= 64) FS_OUT(TT, 4, 4, I, 1, 0); else FS_OUT(TT, 8, 4, I, 2, 0); \
        } else {                                                                                                          \
            if (dim <= 32) FS_OUT(TT, 2, 8, I, 0, 1); else if (dim <= 64) FS_OUT(TT, 4, 8, I, 1, 1); else FS_OUT(TT, 8, 8, I, 2, 1); \
        }                                                                                                                 \
    } while (0)
        if (dtype == IA_F32) FS_BOTH(float, 0);
        else FS_BOTH(bf16_t, 1);
#undef FS_BOTH
#undef FS_OUT
#undef FS_LOCAL
    }
    IA_LAUNCH_CHECK("fading_scan (chunks)");
    return 0;
}
