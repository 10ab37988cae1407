// State-space duality (Mamba-2): a recurrence whose decay is one number a head and token.
//
//     dt_t = softplus(raw_t + dt_bias_h),      a_t = exp(-exp(A_log_h) dt_t)                     (per head, float32)
//     S_t  = a_t S_(t-1) + dt_t B_t x_t^T,     y_t = S_t^T C_t + D_h x_t                         (S: N x P per head, from zero)
//
// with B and C shared by the heads of a group (head h reads group h / (heads / groups)).  Everything is float32.  The
// state of a request is kept column by column, [slots, heads, P, N], so that a column's N values lie side by side.
//
// Two forms: `scan` walks an entry's tokens one by one (decoded tokens, short portions, sizes the other does not take);
// `chunked` cuts a long portion into chunks of 64 tokens whose work is matrix products.
//
// scan.  A workgroup (four wavefronts) owns 4 * 64 / LPC columns of one (entry, head).  LPC neighbouring lanes share a column:
// lane group g of it holds the rows 4 (g + LPC i) .. + 3 for i < Q in registers (rows past N are padding that stays
// zero).  The tokens' B, C and x, their dt and decay go through LDS SSD_STAGE tokens at a time; the next tokens' values
// are asked of memory before the staged ones are worked on.  Per token a lane updates its rows and sums its share of y,
// the shares are added by data-parallel moves inside the column's lanes, always in one order; the lane group that has a
// token's number (modulo LPC) keeps its y, so that a stage's results leave in a few stores.  Every column evolves by
// itself and tokens run in order from the state that earlier steps left, so a prompt cut into portions, or decoded token
// by token, performs the same operations in the same order as the whole prompt in one step.
#include "common.h"

#define SSD_STAGE 16
#define SSD_WAVES 4

typedef __attribute__((ext_vector_type(4))) float ssd_f32x4;

template <int PATTERN> __device__ __forceinline__ float ssd_dpp(float v) {
    return __builtin_bit_cast(float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), PATTERN, 0xF, 0xF, true));
}
// The sum over the LPC (4, 8 or 16) neighbouring lanes that share a column, left in all of them.
template <int LPC> __device__ __forceinline__ float ssd_group_sum(float v) {
    v += ssd_dpp<0xB1>(v);                          // the neighbour in the quad
    v += ssd_dpp<0x4E>(v);                          // the other pair of the quad
    if (LPC == 8) v += ssd_dpp<0x141>(v);           // the other quad of the half row (mirrored)
    if (LPC == 16) {
        v += ssd_dpp<0x124>(v);                     // the quad four lanes on in the row of 16
        v += ssd_dpp<0x128>(v);                     // the pair of quads eight lanes on
    }
    return v;
}
__device__ __forceinline__ float ssd_softplus(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }

// xbc: [n, heads * P + 2 * groups * N] float32, x then B then C, after the convolution; raw: the tokens' dt as
// projected, rows raw_stride apart; y: [n, heads * P] float32.
template <int LPC, int Q>
__global__ void __launch_bounds__(64 * SSD_WAVES)
ssd_scan_kernel(const float* __restrict__ xbc, const float* __restrict__ raw, int64_t raw_stride,
                const float* __restrict__ dt_bias, const float* __restrict__ a_log, const float* __restrict__ d_skip,
                const int* __restrict__ entry_start, const int* __restrict__ state_slots, float* __restrict__ state,
                int heads, int groups, int P, int N, int chunked_from, float* __restrict__ y) {
    constexpr int ROWS = 4 * LPC * Q, WCOLS = 64 / LPC, COLS = SSD_WAVES * WCOLS, NT = 64 * SSD_WAVES;
    constexpr int PIECES = SSD_STAGE * ROWS / NT;            // values of B (and of C) a thread stages
    constexpr int XPIECES = (SSD_STAGE * COLS + NT - 1) / NT;
    static_assert(SSD_STAGE % LPC == 0, "a stage's tokens are dealt to the lane groups evenly");
    __shared__ __attribute__((aligned(16))) float sb[SSD_STAGE][ROWS];
    __shared__ __attribute__((aligned(16))) float sc[SSD_STAGE][ROWS];
    __shared__ float sx[SSD_STAGE][COLS];
    __shared__ float sdt[SSD_STAGE], sa[SSD_STAGE];
    const int e = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int col0 = blockIdx.z * COLS, cidx = wave * WCOLS + lane / LPC, col = col0 + cidx, g = lane % LPC;
    const bool live = col < P;
    const int t0 = entry_start[e], t1 = entry_start[e + 1];
    if (t0 >= t1 || t1 - t0 >= chunked_from) return;         // long entries are the chunked kernels'
    const int C = heads * P + 2 * groups * N, group = h / (heads / groups);
    const float* xs = xbc + (int64_t)h * P + col0;
    const float* bs = xbc + (int64_t)heads * P + (int64_t)group * N;
    const float* cs = bs + (int64_t)groups * N;
    const float rate = expf(a_log[h]), bias = dt_bias[h], skip = d_skip[h];
    float* S = state + (((int64_t)state_slots[e] * heads + h) * P + (live ? col : 0)) * (int64_t)N;
    float s[Q][4];
#pragma unroll
    for (int q = 0; q < Q; ++q)
#pragma unroll
        for (int x = 0; x < 4; ++x) {
            const int n = 4 * (g + LPC * q) + x;
            s[q][x] = live && n < N ? S[n] : 0.f;
        }
    float nb[PIECES], nc[PIECES], nx[XPIECES], nraw = 0.f;
    // addresses are clamped into the entry's rows and the rows' channels; what they bring for padding is dropped when it
    // is staged
    auto fetch = [&](int base) {
#pragma unroll
        for (int j = 0; j < PIECES; ++j) {
            const int i = tid + NT * j;
            const int64_t row = (int64_t)min(base + i / ROWS, t1 - 1) * C + min(i % ROWS, N - 1);
            nb[j] = bs[row];
            nc[j] = cs[row];
        }
#pragma unroll
        for (int j = 0; j < XPIECES; ++j) {
            const int i = tid + NT * j;
            nx[j] = xs[(int64_t)min(base + min(i / COLS, SSD_STAGE - 1), t1 - 1) * C + min(i % COLS, P - 1 - col0)];
        }
        if (tid < SSD_STAGE) nraw = raw[(int64_t)min(base + tid, t1 - 1) * raw_stride + h];
    };
    fetch(t0);
    for (int base = t0; base < t1; base += SSD_STAGE) {
        __syncthreads();                                     // the last stage's reads
#pragma unroll
        for (int j = 0; j < PIECES; ++j) {
            const int i = tid + NT * j;
            sb[i / ROWS][i % ROWS] = i % ROWS < N ? nb[j] : 0.f;
            sc[i / ROWS][i % ROWS] = i % ROWS < N ? nc[j] : 0.f;
        }
#pragma unroll
        for (int j = 0; j < XPIECES; ++j) {
            const int i = tid + NT * j;
            if (i < SSD_STAGE * COLS) sx[i / COLS][i % COLS] = col0 + i % COLS < P ? nx[j] : 0.f;
        }
        if (tid < SSD_STAGE) {
            // a token past the entry's last leaves the state as it is: dt 0, decay 1
            const float dt = base + tid < t1 ? ssd_softplus(nraw + bias) : 0.f;
            sdt[tid] = dt;
            sa[tid] = expf(-rate * dt);
        }
        __syncthreads();
        if (base + SSD_STAGE < t1) fetch(base + SSD_STAGE);
        float keep[SSD_STAGE / LPC];
#pragma unroll
        for (int tt = 0; tt < SSD_STAGE; ++tt) {
            const float a = sa[tt], u = sdt[tt] * sx[tt][cidx];
            float part[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int q = 0; q < Q; ++q) {
                const ssd_f32x4 b4 = *reinterpret_cast<const ssd_f32x4*>(&sb[tt][4 * (g + LPC * q)]);
                const ssd_f32x4 c4 = *reinterpret_cast<const ssd_f32x4*>(&sc[tt][4 * (g + LPC * q)]);
#pragma unroll
                for (int x = 0; x < 4; ++x) {
                    s[q][x] = fmaf(a, s[q][x], b4[x] * u);
                    part[x] = fmaf(s[q][x], c4[x], part[x]);
                }
            }
            const float sum = ssd_group_sum<LPC>((part[0] + part[1]) + (part[2] + part[3]));
            if (g == tt % LPC) keep[tt / LPC] = sum;
        }
#pragma unroll
        for (int k = 0; k < SSD_STAGE / LPC; ++k) {
            const int tt = k * LPC + g;
            if (live && base + tt < t1) y[((int64_t)(base + tt) * heads + h) * P + col] = fmaf(skip, sx[tt][cidx], keep[k]);
        }
    }
    if (!live) return;
#pragma unroll
    for (int q = 0; q < Q; ++q)
#pragma unroll
        for (int x = 0; x < 4; ++x) {
            const int n = 4 * (g + LPC * q) + x;
            if (n < N) S[n] = s[q][x];
        }
}

// ------------------------------------------------------------------------------------------------ in chunks
// With the chunk's first token as number 0, S the state before it and, for tokens i >= j of it, the decay from j to i
// m_ij = a_(j+1) ... a_i and from the chunk's start to i p_i = a_0 ... a_i (products of the tokens' decays, as the scan
// forms them one by one):
//
//     y_i  = p_i S^T C_i + sum_(j <= i) m_ij dt_j (B_j . C_i) x_j + D x_i
//     S'   = p_last S + dS,     dS = sum_j m_(last, j) dt_j B_j x_j^T
//
// Three launches: `local` (dS of every chunk and p_last), `carry` (the states before every chunk, one after another,
// elementwise, and the request's state after the last), `output` (y).  All products are 16 x 16 x 4 float32 matrix
// instructions with operands straight from memory.  A lane l of an instruction supplies A[l % 16][l / 16] and B[l /
// 16][l % 16] and receives D[4 (l / 16) + r][l % 16].  Sums may run over K in any order, and rows and columns may be
// numbered as it suits: where an operand's rows lie along K in memory, a lane reads four values of K at once for four
// instructions; where they lie across, it reads four rows' (or columns') values for four tiles.
#define SSD_CHUNK 64
#define SSD_CHUNKED_FROM 64          // entries of at least this many tokens go through the chunked kernels

struct SsdArgs {
    const float* xbc;                // [n, heads * P + 2 * groups * N]: x, B, C
    const float* raw;                // dt as projected, rows raw_stride apart
    int64_t raw_stride;
    const float* dt_bias;
    const float* a_log;
    const float* d_skip;
    const int* entry_start;
    const int* state_slots;
    float* state;                    // [slots, heads, P, N]
    int heads, groups, P, N;
    float* y;                        // [n, heads * P]
    float* local;                    // [chunks, heads, P, N]: dS of a chunk, then the state before it
    float* decay;                    // [chunks, heads]: p_last
};

__device__ __forceinline__ ssd_f32x4 ssd_mfma(float a, float b, ssd_f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}
// Where the chunks of entry e begin in the workspaces: entries never share a place, whatever their lengths.
__device__ __forceinline__ int64_t ssd_first_chunk(int e, int start) { return start / SSD_CHUNK + e; }

// Lane j's token of the chunk: dt and decay; a token past the entry's last has dt 0 and decay 1.
__device__ __forceinline__ void ssd_token(const SsdArgs& p, int h, int t, int t1, float& dt, float& a) {
    dt = t < t1 ? ssd_softplus(p.raw[(int64_t)t * p.raw_stride + h] + p.dt_bias[h]) : 0.f;
    a = expf(-expf(p.a_log[h]) * dt);
}

// grid (chunks of the longest entry, entries, heads * blocks of 64 p * blocks of 64 n); a wavefront a workgroup.
__global__ void __launch_bounds__(64)
ssd_local_kernel(const SsdArgs p, int p_blocks, int n_blocks) {
    const int e = blockIdx.y, lane = threadIdx.x, c = lane & 15, q = lane >> 4;
    const int start = p.entry_start[e], t1 = p.entry_start[e + 1], base = start + blockIdx.x * SSD_CHUNK;
    if (t1 - start < SSD_CHUNKED_FROM || base >= t1) return;
    const int nb = blockIdx.z % n_blocks, pb = blockIdx.z / n_blocks % p_blocks, h = blockIdx.z / (n_blocks * p_blocks);
    const int C = p.heads * p.P + 2 * p.groups * p.N, group = h / (p.heads / p.groups);
    const int64_t chunk = ssd_first_chunk(e, start) + blockIdx.x;
    float dt, a;
    ssd_token(p, h, base + lane, t1, dt, a);
    float after = a;                                      // the product of the decays of this token and all later ones
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const float other = __shfl_down(after, off, 64);
        if (lane + off < 64) after *= other;
    }
    if (lane == 0 && nb == 0 && pb == 0) p.decay[chunk * p.heads + h] = after;
    const float later = __shfl_down(after, 1, 64);
    const float weight = dt * (lane < 63 ? later : 1.f);
    const int p0 = pb * 64 + 4 * c, n0 = nb * 64 + 4 * c;
    const bool p_live = p0 < p.P, n_live = n0 < p.N;
    const float* xs = p.xbc + (int64_t)h * p.P + (p_live ? p0 : 0);
    const float* bs = p.xbc + (int64_t)p.heads * p.P + (int64_t)group * p.N + (n_live ? n0 : 0);
    ssd_f32x4 acc[4][4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = ssd_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s = 0; s < SSD_CHUNK / 4; ++s) {
        const int64_t row = (int64_t)min(base + 4 * s + q, t1 - 1) * C;
        ssd_f32x4 x4 = *reinterpret_cast<const ssd_f32x4*>(xs + row);
        const ssd_f32x4 b4 = *reinterpret_cast<const ssd_f32x4*>(bs + row);
        x4 *= __shfl(weight, 4 * s + q, 64);
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int j = 0; j < 4; ++j) acc[i][j] = ssd_mfma(x4[i], b4[j], acc[i][j]);
    }
    // tile (i, j), register r: p = 4 (4 q + r) + i, n = 4 c + j
    float* to = p.local + ((chunk * p.heads + h) * p.P) * (int64_t)p.N;
    if (!n_live) return;
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int pp = pb * 64 + 4 * (4 * q + r) + i;
            if (pp < p.P)
                *reinterpret_cast<ssd_f32x4*>(to + (int64_t)pp * p.N + n0) = ssd_f32x4{acc[i][0][r], acc[i][1][r], acc[i][2][r], acc[i][3][r]};
        }
}

// grid (four elements of a head's state a thread, entries, heads)
__global__ void __launch_bounds__(256)
ssd_carry_kernel(const SsdArgs p) {
    const int e = blockIdx.y, h = blockIdx.z;
    const int start = p.entry_start[e], len = p.entry_start[e + 1] - start;
    if (len < SSD_CHUNKED_FROM) return;
    const int64_t size = (int64_t)p.P * p.N, at = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
    if (at >= size) return;
    const int chunks = (len + SSD_CHUNK - 1) / SSD_CHUNK;
    const int64_t first = ssd_first_chunk(e, start), stride = (int64_t)p.heads * size;
    float* kept = p.state + ((int64_t)p.state_slots[e] * p.heads + h) * size + at;
    float* mine = p.local + (first * p.heads + h) * size + at;
    ssd_f32x4 s = *reinterpret_cast<const ssd_f32x4*>(kept);
    for (int k = 0; k < chunks; k += 4) {
        ssd_f32x4 d[4];
        float decay[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {                        // four chunks are asked for before the first is used
            const int kk = min(k + u, chunks - 1);
            d[u] = *reinterpret_cast<const ssd_f32x4*>(mine + kk * stride);
            decay[u] = p.decay[(first + kk) * p.heads + h];
        }
#pragma unroll
        for (int u = 0; u < 4; ++u)
            if (k + u < chunks) {
                *reinterpret_cast<ssd_f32x4*>(mine + (k + u) * stride) = s;
#pragma unroll
                for (int x = 0; x < 4; ++x) s[x] = fmaf(decay[u], s[x], d[u][x]);
            }
    }
    *reinterpret_cast<ssd_f32x4*>(kept) = s;
}

// grid (chunks of the longest entry, entries, heads * blocks of 64 p).  Wavefront w of the four owns the tokens 16 w ..
// 16 w + 15 of the chunk and computes y transposed: rows p, columns its tokens.  NS: ceil(N / 16), at least N / 16.
template <int NS>
__global__ void __launch_bounds__(256)
ssd_output_kernel(const SsdArgs p, int p_blocks) {
    __shared__ __attribute__((aligned(16))) float m_s[4][16][SSD_CHUNK + 4];      // a wavefront's own: [token][j], m_ij dt_j
    const int e = blockIdx.y, lane = threadIdx.x & 63, w = threadIdx.x >> 6, c = lane & 15, q = lane >> 4;
    const int start = p.entry_start[e], t1 = p.entry_start[e + 1], base = start + blockIdx.x * SSD_CHUNK;
    if (t1 - start < SSD_CHUNKED_FROM || base + 16 * w >= t1) return;             // no barrier below: wavefronts are on their own
    const int pb = blockIdx.z % p_blocks, h = blockIdx.z / p_blocks;
    const int C = p.heads * p.P + 2 * p.groups * p.N, group = h / (p.heads / p.groups);
    const int64_t chunk = ssd_first_chunk(e, start) + blockIdx.x;
    float dt, a;
    ssd_token(p, h, base + lane, t1, dt, a);
    // lane j: m_ij dt_j for the wavefront's tokens i (0 for i < j), as running products; and p_i of the lane's own token
    float m = 1.f, run = 1.f, from_start = 1.f;
#pragma unroll
    for (int k = 0; k < SSD_CHUNK; ++k) {
        if (k > 16 * w + 15) break;
        const float ak = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(a), k));
        run *= ak;
        if (k == 16 * w + c) from_start = run;
        m = k > lane ? m * ak : 1.f;
        if (k >= 16 * w) m_s[w][k - 16 * w][lane] = k >= lane ? m * dt : 0.f;
    }
    __builtin_amdgcn_wave_barrier();                         // a wavefront's LDS stores and reads are in order
    const int ti = min(base + 16 * w + c, t1 - 1);           // the lane's token (clamped: what it brings is not stored)
    const float* bs = p.xbc + (int64_t)p.heads * p.P + (int64_t)group * p.N + 4 * q;
    const float* cs = bs + (int64_t)p.groups * p.N + (int64_t)ti * C;
    ssd_f32x4 cf[NS];
#pragma unroll
    for (int s = 0; s < NS; ++s)
        cf[s] = 16 * s + 4 * q < p.N ? *reinterpret_cast<const ssd_f32x4*>(cs + 16 * s) : ssd_f32x4{0.f, 0.f, 0.f, 0.f};
    // tile i holds the rows p = 64 pb + 4 r + i; an operand's row past P is some other row, whose result is not stored
    ssd_f32x4 acc[4];
    const float* ss = p.local + ((chunk * p.heads + h) * p.P) * (int64_t)p.N + 4 * q;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        acc[i] = ssd_f32x4{0.f, 0.f, 0.f, 0.f};
        const float* row = ss + (int64_t)min(pb * 64 + 4 * c + i, p.P - 1) * p.N;
#pragma unroll
        for (int s = 0; s < NS; ++s) {
            const ssd_f32x4 s4 = 16 * s + 4 * q < p.N ? *reinterpret_cast<const ssd_f32x4*>(row + 16 * s) : ssd_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int x = 0; x < 4; ++x) acc[i] = ssd_mfma(s4[x], cf[s][x], acc[i]);
        }
        acc[i] *= from_start;
    }
    const int p0 = pb * 64 + 4 * c;
    const float* xs = p.xbc + (int64_t)h * p.P + (p0 < p.P ? p0 : 0);
    for (int jt = 0; jt <= w; ++jt) {
        // (B_j . C_i) for j = 16 jt + row, i = the lane's token; its register r is j = 16 jt + 4 q + r: what the next
        // product takes as its K values 4 q + r
        ssd_f32x4 g = {0.f, 0.f, 0.f, 0.f};
        const float* brow = bs + (int64_t)min(base + 16 * jt + c, t1 - 1) * C;
        ssd_f32x4 xf[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) xf[r] = *reinterpret_cast<const ssd_f32x4*>(xs + (int64_t)min(base + 16 * jt + 4 * q + r, t1 - 1) * C);
#pragma unroll
        for (int s = 0; s < NS; ++s) {
            const ssd_f32x4 b4 = 16 * s + 4 * q < p.N ? *reinterpret_cast<const ssd_f32x4*>(brow + 16 * s) : ssd_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int x = 0; x < 4; ++x) g = ssd_mfma(b4[x], cf[s][x], g);
        }
        g *= *reinterpret_cast<const ssd_f32x4*>(&m_s[w][c][16 * jt + 4 * q]);
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
            for (int i = 0; i < 4; ++i) acc[i] = ssd_mfma(xf[r][i], g[r], acc[i]);
    }
    if (base + 16 * w + c >= t1) return;
    const float skip = p.d_skip[h];
    const float* xi = p.xbc + (int64_t)ti * C + (int64_t)h * p.P;
    float* yi = p.y + ((int64_t)ti * p.heads + h) * p.P;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int pp = pb * 64 + 16 * q + 4 * r;             // four neighbours, one of each tile
        if (pp >= p.P) continue;
        const ssd_f32x4 x4 = *reinterpret_cast<const ssd_f32x4*>(xi + pp);
        *reinterpret_cast<ssd_f32x4*>(yi + pp) = ssd_f32x4{fmaf(skip, x4[0], acc[0][r]), fmaf(skip, x4[1], acc[1][r]),
                                                           fmaf(skip, x4[2], acc[2][r]), fmaf(skip, x4[3], acc[3][r])};
    }
}

// Whether the chunked kernels take these sizes (four neighbours of a row at a time).
extern "C" int somi_ssd_chunked(int P, int N) { return P % 4 == 0 && N % 4 == 0 && N <= 256; }
// Places of a chunk that the workspaces of a step hold, and the shortest entry that uses them.
extern "C" int64_t somi_ssd_chunks(int n_tokens, int n_entries) { return (int64_t)n_tokens / SSD_CHUNK + n_entries + 1; }
extern "C" int somi_ssd_chunked_from() { return SSD_CHUNKED_FROM; }

// max_entry_len: the longest entry.  local, decay: workspaces of somi_ssd_chunks(n_tokens, n_entries) * heads * P * N and
// * heads floats, or null: then every entry is scanned.  one_entry != 0: the step holds a single entry.
extern "C" int somi_ssd(const float* xbc, const float* raw, int64_t raw_stride, const float* dt_bias, const float* a_log,
                        const float* d_skip, const int* entry_start, const int* state_slots, float* state, int n_entries,
                        int max_entry_len, int heads, int groups, int P, int N, float* local, float* decay, float* y,
                        hipStream_t stream) {
    SOMI_REQUIRE(n_entries >= 0 && max_entry_len >= 0 && heads > 0 && groups > 0 && heads % groups == 0 && P > 0 && N > 0, "ssd: bad sizes");
    SOMI_REQUIRE(N <= 512, "ssd: a state of %d rows is more than the supported 512", N);
    SOMI_REQUIRE(raw_stride >= heads, "ssd: rows too narrow");
    if (n_entries == 0) return 0;
    const bool chunked = local != nullptr && max_entry_len >= SSD_CHUNKED_FROM;
    if (!(chunked && n_entries == 1)) {
        // lanes a column: from the model's sizes only, so that a request's sums have one order in every batch
        const int lpc = N <= 16 ? 4 : N <= 32 ? 8 : 16;
        const int q = ceil_div(N, 4 * lpc), cols = SSD_WAVES * 64 / lpc;
        SOMI_REQUIRE(heads <= 65535 && ceil_div(P, cols) <= 65535, "ssd: too many heads or columns");
        const dim3 grid(n_entries, heads, ceil_div(P, cols));
        const int from = chunked ? SSD_CHUNKED_FROM : 0x7fffffff;
#define SOMI_SSD(L, QQ)                                                                                                      \
    hipLaunchKernelGGL((ssd_scan_kernel<L, QQ>), grid, dim3(64 * SSD_WAVES), 0, stream, xbc, raw, raw_stride, dt_bias, a_log, \
                       d_skip, entry_start, state_slots, state, heads, groups, P, N, from, y)
        if (lpc == 4) SOMI_SSD(4, 1);
        else if (lpc == 8) SOMI_SSD(8, 1);
        else if (q <= 1) SOMI_SSD(16, 1);
        else if (q <= 2) SOMI_SSD(16, 2);
        else if (q <= 3) SOMI_SSD(16, 3);
        else if (q <= 4) SOMI_SSD(16, 4);
        else SOMI_SSD(16, 8);
#undef SOMI_SSD
        SOMI_LAUNCH_CHECK("ssd_scan");
    }
    if (!chunked) return 0;
    SOMI_REQUIRE(somi_ssd_chunked(P, N), "ssd: heads of %d with a state of %d rows are not what the chunked kernels are built for", P, N);
    SOMI_REQUIRE(decay != nullptr && (uintptr_t)xbc % 16 == 0 && (uintptr_t)state % 16 == 0 && (uintptr_t)local % 16 == 0 && (uintptr_t)y % 16 == 0,
                 "ssd: operands must be aligned to 16 bytes");
    const int chunks = ceil_div(max_entry_len, SSD_CHUNK), p_blocks = ceil_div(P, 64), n_blocks = ceil_div(N, 64);
    SOMI_REQUIRE(n_entries <= 65535 && heads * p_blocks * n_blocks <= 65535, "ssd: too many entries or heads");
    const SsdArgs args{xbc, raw, raw_stride, dt_bias, a_log, d_skip, entry_start, state_slots, state, heads, groups, P, N, y, local, decay};
    hipLaunchKernelGGL(ssd_local_kernel, dim3(chunks, n_entries, heads * p_blocks * n_blocks), dim3(64), 0, stream, args, p_blocks, n_blocks);
    SOMI_LAUNCH_CHECK("ssd_local");
    hipLaunchKernelGGL(ssd_carry_kernel, dim3((unsigned)ceil_div64((int64_t)P * N, 1024), n_entries, heads), dim3(256), 0, stream, args);
    SOMI_LAUNCH_CHECK("ssd_carry");
    const dim3 grid(chunks, n_entries, heads * p_blocks);
#define SOMI_SSD_OUT(NS) hipLaunchKernelGGL(ssd_output_kernel<NS>, grid, dim3(256), 0, stream, args, p_blocks)
    if (N <= 16) SOMI_SSD_OUT(1);
    else if (N <= 32) SOMI_SSD_OUT(2);
    else if (N <= 64) SOMI_SSD_OUT(4);
    else if (N <= 128) SOMI_SSD_OUT(8);
    else SOMI_SSD_OUT(16);
#undef SOMI_SSD_OUT
    SOMI_LAUNCH_CHECK("ssd_output");
    return 0;
}

// ------------------------------------------------------------------------------------------------ gate and norm
// u = y * silu(z), RMS-normed in `groups` equal parts of a row (eps inside the root), times w and `scale`.  A
// workgroup a (token, part).  y: [n, width] float32; z: float32, rows z_stride apart; out: rows of `width`, out_stride
// apart.
template <typename T>
__global__ void __launch_bounds__(256)
gated_group_norm_kernel(const float* __restrict__ y, const float* __restrict__ z, int64_t z_stride,
                        const float* __restrict__ w, float eps, float scale, int width, int part, T* __restrict__ out,
                        int64_t out_stride) {
    __shared__ float red[16];
    const int64_t t = blockIdx.x;
    const int at = blockIdx.y * part;
    const float* yr = y + t * width + at;
    const float* zr = z + t * z_stride + at;
    constexpr int HELD = 16;                  // values a thread keeps between the sum and the scaling
    float held[HELD], ss = 0.f;
    auto value = [&](int c) {
        const float gate = zr[c];
        return yr[c] * (gate / (1.0f + expf(-gate)));
    };
#pragma unroll
    for (int j = 0; j < HELD; ++j) {
        if (256 * j >= part) break;                      // the same for the whole workgroup
        const int c = threadIdx.x + 256 * j;
        const float v = value(min(c, part - 1));
        held[j] = c < part ? v : 0.f;
        ss = fmaf(held[j], held[j], ss);
    }
    for (int c = threadIdx.x + 256 * HELD; c < part; c += 256) {
        const float v = value(c);
        ss = fmaf(v, v, ss);
    }
    ss = block_sum<256>(ss, red);
    const float inv = scale / sqrtf(ss / (float)part + eps);
    T* to = out + t * out_stride + at;
#pragma unroll
    for (int j = 0; j < HELD; ++j) {
        const int c = threadIdx.x + 256 * j;
        if (c < part) to[c] = from_float<T>(held[j] * inv * w[at + c]);
    }
    for (int c = threadIdx.x + 256 * HELD; c < part; c += 256) to[c] = from_float<T>(value(c) * inv * w[at + c]);
}

extern "C" int somi_gated_group_norm(const float* y, const float* z, int64_t z_stride, const float* w, int groups, float eps,
                                     float scale, int n_tokens, int width, void* out, int64_t out_stride, int dtype,
                                     hipStream_t stream) {
    SOMI_REQUIRE(n_tokens >= 0 && width > 0 && groups > 0 && width % groups == 0, "gated_group_norm: %d values in %d parts", width, groups);
    SOMI_REQUIRE(z_stride >= width && out_stride >= width && groups <= 65535, "gated_group_norm: bad strides");
    if (n_tokens == 0) return 0;
    const dim3 grid(n_tokens, groups);
    if (dtype == SOMI_F32)
        hipLaunchKernelGGL(gated_group_norm_kernel<float>, grid, dim3(256), 0, stream, y, z, z_stride, w, eps, scale, width,
                           width / groups, (float*)out, out_stride);
    else if (dtype == SOMI_BF16)
        hipLaunchKernelGGL(gated_group_norm_kernel<bf16>, grid, dim3(256), 0, stream, y, z, z_stride, w, eps, scale, width,
                           width / groups, (bf16*)out, out_stride);
    else
        return somi_fail("gated_group_norm: unknown dtype %d", dtype);
    SOMI_LAUNCH_CHECK("gated_group_norm");
    return 0;
}
