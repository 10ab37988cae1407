// Linear recurrences whose decay is one number a head and token, with a matrix state a head:
//
//     S_t = a_t S_(t-1) + w_t B_t x_t^T,     y_t = scale S_t^T C_t + D_h x_t                     (S: N x P per head, from zero)
//
// with B and C shared by the heads of a group (head h reads group h / (heads / groups)).  Where a_t and w_t come from:
//
//     SSD_DT      w_t = softplus(raw_t + dt_bias_h),  a_t = exp(-exp(A_log_h) w_t)               (Mamba-2; the only one with a D)
//     SSD_GIVEN   both given for every token and head                                            (mLSTM: csrc/mlstm.hip makes them)
//     SSD_FIXED   a_t = decay_h,  w_t = 1                                                        (lightning attention)
//
// With a normaliser a head also keeps n_t = a_t n_(t-1) + w_t B_t and gives den_t = scale n_t . C_t: one more column of
// the state, whose x is 1.  Everything is float32.  The state of a request is kept column by column, [slots, heads, P (+ 1),
// N], so that a column's N values lie side by side; the normaliser is the last column.
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

enum SsdKind { SSD_DT = 0, SSD_GIVEN = 1, SSD_FIXED = 2 };

struct SsdArgs {
    const float* x;                  // the tokens' rows, row_stride apart: head h's x at h * P,
    const float* b;                  // group g's B at g * N
    const float* c;                  // and its C at g * N
    int64_t row_stride;
    const float* raw;                // SSD_DT: dt as projected, rows raw_stride apart
    int64_t raw_stride;
    const float* dt_bias;
    const float* a_log;
    const float* d_skip;
    const float* keep;               // SSD_GIVEN: a_t, [n, heads]; SSD_FIXED: the decays, [heads]
    const float* write;              // SSD_GIVEN: w_t, [n, heads]
    float scale;
    const int* entry_start;
    const int* state_slots;
    float* state;                    // [slots, heads, P (+ 1), N]
    int heads, groups, P, N;
    float* y;                        // [n, heads * P]
    float* den;                      // with a normaliser: [n, heads]
    float* local;                    // [chunks, heads, P (+ 1), N]: dS of a chunk, then the state before it
    float* decay;                    // [chunks, heads]: p_last
};

// Token t's decay and write weight; a token past the entry's last leaves the state as it is (decay 1, weight 0).
template <int KIND>
__device__ __forceinline__ void ssd_token(const SsdArgs& p, int h, int t, int t1, float& w, float& a) {
    if (KIND == SSD_DT) {
        w = t < t1 ? ssd_softplus(p.raw[(int64_t)t * p.raw_stride + h] + p.dt_bias[h]) : 0.f;
        a = expf(-expf(p.a_log[h]) * w);
    } else if (KIND == SSD_GIVEN) {
        w = t < t1 ? p.write[(int64_t)t * p.heads + h] : 0.f;
        a = t < t1 ? p.keep[(int64_t)t * p.heads + h] : 1.f;
    } else {
        w = t < t1 ? 1.f : 0.f;
        a = t < t1 ? p.keep[h] : 1.f;
    }
}

template <int LPC, int Q, int KIND, bool NORM>
__global__ void __launch_bounds__(64 * SSD_WAVES)
ssd_scan_kernel(const SsdArgs p, int chunked_from) {
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
    const int heads = p.heads, P = p.P, N = p.N, PR = P + (NORM ? 1 : 0);
    const bool live = col < PR;
    const int t0 = p.entry_start[e], t1 = p.entry_start[e + 1];
    if (t0 >= t1 || t1 - t0 >= chunked_from) return;         // long entries are the chunked kernels'
    const int64_t C = p.row_stride;
    const int group = h / (heads / p.groups);
    const float* xs = p.x + (int64_t)h * P + col0;
    const float* bs = p.b + (int64_t)group * N;
    const float* cs = p.c + (int64_t)group * N;
    const float skip = KIND == SSD_DT ? p.d_skip[h] : 0.f;
    float* S = p.state + (((int64_t)p.state_slots[e] * heads + h) * PR + (live ? col : 0)) * (int64_t)N;
    float s[Q][4];
#pragma unroll
    for (int q = 0; q < Q; ++q)
#pragma unroll
        for (int x = 0; x < 4; ++x) {
            const int n = 4 * (g + LPC * q) + x;
            s[q][x] = live && n < N ? S[n] : 0.f;
        }
    float nb[PIECES], nc[PIECES], nx[XPIECES], nw = 0.f, na = 1.f;
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
        if (tid < SSD_STAGE) ssd_token<KIND>(p, h, base + tid, t1, nw, na);
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
            if (i < SSD_STAGE * COLS) sx[i / COLS][i % COLS] = col0 + i % COLS < P ? nx[j] : (NORM && col0 + i % COLS == P ? 1.f : 0.f);
        }
        if (tid < SSD_STAGE) {
            sdt[tid] = nw;
            sa[tid] = na;
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
            if (!live || base + tt >= t1) continue;
            const int64_t at = (int64_t)(base + tt) * heads + h;
            if (NORM && col == P) p.den[at] = p.scale * keep[k];
            else p.y[at * P + col] = KIND == SSD_DT ? fmaf(skip, sx[tt][cidx], p.scale * keep[k]) : p.scale * keep[k];
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
//     y_i  = p_i S^T C_i + sum_(j <= i) m_ij w_j (B_j . C_i) x_j + D x_i
//     S'   = p_last S + dS,     dS = sum_j m_(last, j) w_j B_j x_j^T
//
// (the normaliser's column, whose x is 1, takes row sums of what the two products hold already).
//
// Three launches: `local` (dS of every chunk and p_last), `carry` (the states before every chunk, one after another,
// elementwise, and the request's state after the last), `output` (y).  All products are 16 x 16 x 4 float32 matrix
// instructions with operands straight from memory.  A lane l of an instruction supplies A[l % 16][l / 16] and B[l /
// 16][l % 16] and receives D[4 (l / 16) + r][l % 16].  Sums may run over K in any order, and rows and columns may be
// numbered as it suits: where an operand's rows lie along K in memory, a lane reads four values of K at once for four
// instructions; where they lie across, it reads four rows' (or columns') values for four tiles.
#define SSD_CHUNK 64
#define SSD_CHUNKED_FROM 64          // entries of at least this many tokens go through the chunked kernels

__device__ __forceinline__ ssd_f32x4 ssd_mfma(float a, float b, ssd_f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}
// Where the chunks of entry e begin in the workspaces: entries never share a place, whatever their lengths.
__device__ __forceinline__ int64_t ssd_first_chunk(int e, int start) { return start / SSD_CHUNK + e; }

// grid (chunks of the longest entry, entries, heads * blocks of 64 p * blocks of 64 n); a wavefront a workgroup.
template <int KIND, bool NORM>
__global__ void __launch_bounds__(64)
ssd_local_kernel(const SsdArgs p, int p_blocks, int n_blocks) {
    const int e = blockIdx.y, lane = threadIdx.x, c = lane & 15, q = lane >> 4;
    const int start = p.entry_start[e], t1 = p.entry_start[e + 1], base = start + blockIdx.x * SSD_CHUNK;
    if (t1 - start < SSD_CHUNKED_FROM || base >= t1) return;
    const int nb = blockIdx.z % n_blocks, pb = blockIdx.z / n_blocks % p_blocks, h = blockIdx.z / (n_blocks * p_blocks);
    const int64_t C = p.row_stride;
    const int group = h / (p.heads / p.groups), PR = p.P + (NORM ? 1 : 0);
    const int64_t chunk = ssd_first_chunk(e, start) + blockIdx.x;
    float dt, a;
    ssd_token<KIND>(p, h, base + lane, t1, dt, a);
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
    const float* xs = p.x + (int64_t)h * p.P + (p_live ? p0 : 0);
    const float* bs = p.b + (int64_t)group * p.N + (n_live ? n0 : 0);
    ssd_f32x4 acc[4][4], norm = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = ssd_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s = 0; s < SSD_CHUNK / 4; ++s) {
        const int64_t row = (int64_t)min(base + 4 * s + q, t1 - 1) * C;
        ssd_f32x4 x4 = *reinterpret_cast<const ssd_f32x4*>(xs + row);
        const ssd_f32x4 b4 = *reinterpret_cast<const ssd_f32x4*>(bs + row);
        const float weigh = __shfl(weight, 4 * s + q, 64);
        x4 *= weigh;
        if (NORM) norm += b4 * weigh;
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int j = 0; j < 4; ++j) acc[i][j] = ssd_mfma(x4[i], b4[j], acc[i][j]);
    }
    // tile (i, j), register r: p = 4 (4 q + r) + i, n = 4 c + j
    float* to = p.local + ((chunk * p.heads + h) * PR) * (int64_t)p.N;
    if (NORM && pb == 0) {                                // lanes 16 apart hold other tokens' shares of the same n
#pragma unroll
        for (int x = 0; x < 4; ++x) {
            norm[x] += __shfl_xor(norm[x], 16, 64);
            norm[x] += __shfl_xor(norm[x], 32, 64);
        }
        if (q == 0 && n_live) *reinterpret_cast<ssd_f32x4*>(to + (int64_t)p.P * p.N + n0) = norm;
    }
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
ssd_carry_kernel(const SsdArgs p, int rows /* P, with a normaliser P + 1 */) {
    const int e = blockIdx.y, h = blockIdx.z;
    const int start = p.entry_start[e], len = p.entry_start[e + 1] - start;
    if (len < SSD_CHUNKED_FROM) return;
    const int64_t size = (int64_t)rows * p.N, at = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
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
template <int NS, int KIND, bool NORM>
__global__ void __launch_bounds__(256)
ssd_output_kernel(const SsdArgs p, int p_blocks) {
    __shared__ __attribute__((aligned(16))) float m_s[4][16][SSD_CHUNK + 4];      // a wavefront's own: [token][j], m_ij dt_j
    const int e = blockIdx.y, lane = threadIdx.x & 63, w = threadIdx.x >> 6, c = lane & 15, q = lane >> 4;
    const int start = p.entry_start[e], t1 = p.entry_start[e + 1], base = start + blockIdx.x * SSD_CHUNK;
    if (t1 - start < SSD_CHUNKED_FROM || base + 16 * w >= t1) return;             // no barrier below: wavefronts are on their own
    const int pb = blockIdx.z % p_blocks, h = blockIdx.z / p_blocks;
    const int64_t C = p.row_stride;
    const int group = h / (p.heads / p.groups), PR = p.P + (NORM ? 1 : 0);
    const int64_t chunk = ssd_first_chunk(e, start) + blockIdx.x;
    float dt, a;
    ssd_token<KIND>(p, h, base + lane, t1, dt, a);
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
    const float* bs = p.b + (int64_t)group * p.N + 4 * q;
    const float* cs = p.c + (int64_t)group * p.N + 4 * q + (int64_t)ti * C;
    ssd_f32x4 cf[NS];
#pragma unroll
    for (int s = 0; s < NS; ++s)
        cf[s] = 16 * s + 4 * q < p.N ? *reinterpret_cast<const ssd_f32x4*>(cs + 16 * s) : ssd_f32x4{0.f, 0.f, 0.f, 0.f};
    // tile i holds the rows p = 64 pb + 4 r + i; an operand's row past P is some other row, whose result is not stored
    ssd_f32x4 acc[4];
    const float* ss = p.local + ((chunk * p.heads + h) * PR) * (int64_t)p.N + 4 * q;
    float den = 0.f;                                         // the lane's share of its token's n . C
    if (NORM && pb == 0) {
#pragma unroll
        for (int s = 0; s < NS; ++s)
            if (16 * s + 4 * q < p.N) {
                const ssd_f32x4 n4 = *reinterpret_cast<const ssd_f32x4*>(ss + (int64_t)p.P * p.N + 16 * s) * cf[s];
                den += (n4[0] + n4[1]) + (n4[2] + n4[3]);
            }
        den *= from_start;
    }
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
    const float* xs = p.x + (int64_t)h * p.P + (p0 < p.P ? p0 : 0);
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
        if (NORM) den += (g[0] + g[1]) + (g[2] + g[3]);
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
            for (int i = 0; i < 4; ++i) acc[i] = ssd_mfma(xf[r][i], g[r], acc[i]);
    }
    if (NORM && pb == 0) {                                   // the shares of the lanes 16 apart: other j, other rows of n
        den += __shfl_xor(den, 16, 64);
        den += __shfl_xor(den, 32, 64);
    }
    if (base + 16 * w + c >= t1) return;
    if (NORM && pb == 0 && q == 0) p.den[(int64_t)ti * p.heads + h] = p.scale * den;
    const float skip = KIND == SSD_DT ? p.d_skip[h] : 0.f;
    const float* xi = p.x + (int64_t)ti * C + (int64_t)h * p.P;
    float* yi = p.y + ((int64_t)ti * p.heads + h) * p.P;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int pp = pb * 64 + 16 * q + 4 * r;             // four neighbours, one of each tile
        if (pp >= p.P) continue;
        ssd_f32x4 out = ssd_f32x4{acc[0][r], acc[1][r], acc[2][r], acc[3][r]} * p.scale;
        if (KIND == SSD_DT) {
            const ssd_f32x4 x4 = *reinterpret_cast<const ssd_f32x4*>(xi + pp);
#pragma unroll
            for (int x = 0; x < 4; ++x) out[x] = fmaf(skip, x4[x], out[x]);
        }
        *reinterpret_cast<ssd_f32x4*>(yi + pp) = out;
    }
}

// Whether the chunked kernels take these sizes (four neighbours of a row at a time).
extern "C" int somi_ssd_chunked(int P, int N) { return P % 4 == 0 && N % 4 == 0 && N <= 256; }
// Places of a chunk that the workspaces of a step hold, and the shortest entry that uses them.
extern "C" int64_t somi_ssd_chunks(int n_tokens, int n_entries) { return (int64_t)n_tokens / SSD_CHUNK + n_entries + 1; }
extern "C" int somi_ssd_chunked_from() { return SSD_CHUNKED_FROM; }

template <int KIND, bool NORM>
static int ssd_launch(const SsdArgs& args, int n_entries, int max_entry_len, hipStream_t stream) {
    const int heads = args.heads, groups = args.groups, P = args.P, N = args.N, rows = P + (NORM ? 1 : 0);
    SOMI_REQUIRE(n_entries >= 0 && max_entry_len >= 0 && heads > 0 && groups > 0 && heads % groups == 0 && P > 0 && N > 0, "ssd: bad sizes");
    SOMI_REQUIRE(N <= 512, "ssd: a state of %d rows is more than the supported 512", N);
    SOMI_REQUIRE(!NORM || args.den != nullptr, "ssd: a normaliser needs a place for its products");
    if (n_entries == 0) return 0;
    const bool chunked = args.local != nullptr && max_entry_len >= SSD_CHUNKED_FROM;
    if (!(chunked && n_entries == 1)) {
        // lanes a column: from the model's sizes only, so that a request's sums have one order in every batch
        const int lpc = N <= 16 ? 4 : N <= 32 ? 8 : 16;
        const int q = ceil_div(N, 4 * lpc), cols = SSD_WAVES * 64 / lpc;
        SOMI_REQUIRE(heads <= 65535 && ceil_div(rows, cols) <= 65535, "ssd: too many heads or columns");
        const dim3 grid(n_entries, heads, ceil_div(rows, cols));
        const int from = chunked ? SSD_CHUNKED_FROM : 0x7fffffff;
#define SOMI_SSD(L, QQ) hipLaunchKernelGGL((ssd_scan_kernel<L, QQ, KIND, NORM>), grid, dim3(64 * SSD_WAVES), 0, stream, args, from)
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
    SOMI_REQUIRE(args.decay != nullptr && (uintptr_t)args.x % 16 == 0 && (uintptr_t)args.b % 16 == 0 && (uintptr_t)args.c % 16 == 0 &&
                     args.row_stride % 4 == 0 && (uintptr_t)args.state % 16 == 0 && (uintptr_t)args.local % 16 == 0 && (uintptr_t)args.y % 16 == 0,
                 "ssd: operands must be aligned to 16 bytes");
    const int chunks = ceil_div(max_entry_len, SSD_CHUNK), p_blocks = ceil_div(P, 64), n_blocks = ceil_div(N, 64);
    SOMI_REQUIRE(n_entries <= 65535 && heads * p_blocks * n_blocks <= 65535, "ssd: too many entries or heads");
    hipLaunchKernelGGL((ssd_local_kernel<KIND, NORM>), dim3(chunks, n_entries, heads * p_blocks * n_blocks), dim3(64), 0, stream, args,
                       p_blocks, n_blocks);
    SOMI_LAUNCH_CHECK("ssd_local");
    hipLaunchKernelGGL(ssd_carry_kernel, dim3((unsigned)ceil_div64((int64_t)rows * N, 1024), n_entries, heads), dim3(256), 0, stream, args, rows);
    SOMI_LAUNCH_CHECK("ssd_carry");
    const dim3 grid(chunks, n_entries, heads * p_blocks);
#define SOMI_SSD_OUT(NS) hipLaunchKernelGGL((ssd_output_kernel<NS, KIND, NORM>), grid, dim3(256), 0, stream, args, p_blocks)
    if (N <= 16) SOMI_SSD_OUT(1);
    else if (N <= 32) SOMI_SSD_OUT(2);
    else if (N <= 64) SOMI_SSD_OUT(4);
    else if (N <= 128) SOMI_SSD_OUT(8);
    else SOMI_SSD_OUT(16);
#undef SOMI_SSD_OUT
    SOMI_LAUNCH_CHECK("ssd_output");
    return 0;
}

// Mamba-2.  xbc: [n, heads * P + 2 * groups * N] float32, x then B then C, after the convolution; raw: the tokens' dt as
// projected, rows raw_stride apart; y: [n, heads * P] float32.
// max_entry_len: the longest entry.  local, decay: workspaces of somi_ssd_chunks(n_tokens, n_entries) * heads * P * N and
// * heads floats, or null: then every entry is scanned.
extern "C" int somi_ssd(const float* xbc, const float* raw, int64_t raw_stride, const float* dt_bias, const float* a_log,
                        const float* d_skip, const int* entry_start, const int* state_slots, float* state, int n_entries,
                        int max_entry_len, int heads, int groups, int P, int N, float* local, float* decay, float* y,
                        hipStream_t stream) {
    SOMI_REQUIRE(raw_stride >= heads, "ssd: rows too narrow");
    SsdArgs args{};
    args.x = xbc;
    args.b = xbc + (int64_t)heads * P;
    args.c = args.b + (int64_t)groups * N;
    args.row_stride = (int64_t)heads * P + 2 * (int64_t)groups * N;
    args.raw = raw;
    args.raw_stride = raw_stride;
    args.dt_bias = dt_bias;
    args.a_log = a_log;
    args.d_skip = d_skip;
    args.scale = 1.f;
    args.entry_start = entry_start;
    args.state_slots = state_slots;
    args.state = state;
    args.heads = heads;
    args.groups = groups;
    args.P = P;
    args.N = N;
    args.y = y;
    args.local = local;
    args.decay = decay;
    return ssd_launch<SSD_DT, false>(args, n_entries, max_entry_len, stream);
}

// The recurrence with decays that are given: k (B), q (C) and v (x) are columns of rows row_stride apart, head h's at h * N
// and h * P.  With `write`: keep and write are a_t and w_t, [n, heads], and there is a normaliser, whose products go to den
// [n, heads]; without: keep holds the heads' fixed decays, [heads], and w_t is 1.  state: [slots, heads, P (+ 1), N]; local
// as somi_ssd's, with P + 1 for P where there is a normaliser.
extern "C" int somi_ssd_memory(const float* q, const float* k, const float* v, int64_t row_stride, const float* keep,
                               const float* write, float scale, const int* entry_start, const int* state_slots, float* state,
                               int n_entries, int max_entry_len, int heads, int P, int N, float* local, float* decay, float* y,
                               float* den, hipStream_t stream) {
    SOMI_REQUIRE(keep != nullptr, "ssd_memory: no decays");
    SsdArgs args{};
    args.x = v;
    args.b = k;
    args.c = q;
    args.row_stride = row_stride;
    args.keep = keep;
    args.write = write;
    args.scale = scale;
    args.entry_start = entry_start;
    args.state_slots = state_slots;
    args.state = state;
    args.heads = heads;
    args.groups = heads;
    args.P = P;
    args.N = N;
    args.y = y;
    args.den = den;
    args.local = local;
    args.decay = decay;
    if (write != nullptr) return ssd_launch<SSD_GIVEN, true>(args, n_entries, max_entry_len, stream);
    return ssd_launch<SSD_FIXED, false>(args, n_entries, max_entry_len, stream);
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

// out = scale * w * (u / rms(u)) * sigmoid(g), the root mean square taken over each of `groups` equal parts of a row (eps
// inside the root).  u = y, or with a normaliser u = y / (max(|den|, floor) + 1e-6), den and floor one number a row and part.
// y: [n, width] float32; g: float32, rows g_stride apart; out: rows of `width`, out_stride apart.  LANES threads a (token,
// part), V neighbouring values at a time.
template <typename T, int LANES, int V>
__global__ void __launch_bounds__(256)
norm_sigmoid_gate_kernel(const float* __restrict__ y, const float* __restrict__ den, const float* __restrict__ floor_,
                         const float* __restrict__ g, int64_t g_stride, const float* __restrict__ w, float eps, float scale,
                         int groups, int width, int part, int64_t units, T* __restrict__ out, int64_t out_stride) {
    typedef __attribute__((ext_vector_type(V))) float vec;
    typedef __attribute__((ext_vector_type(V))) T tvec;
    __shared__ float red[16];
    constexpr int HELD = 4;
    const int64_t unit = LANES == 256 ? (int64_t)blockIdx.x : (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (LANES == 64 && unit >= units) return;               // a wavefront on its own: no barrier below
    const int64_t t = unit / groups;
    const int at = (int)(unit % groups) * part, lane = threadIdx.x % LANES;
    const float* yr = y + t * width + at;
    const float* gr = g + t * g_stride + at;
    const float inv_size = den != nullptr ? 1.0f / (fmaxf(fabsf(den[unit]), floor_[unit]) + 1e-6f) : 1.0f;
    vec held[HELD];
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < HELD; ++j) {
        const int c = V * (lane + LANES * j);
        held[j] = 0.f;
        if (c < part) held[j] = *reinterpret_cast<const vec*>(yr + c) * inv_size;
#pragma unroll
        for (int x = 0; x < V; ++x) ss = fmaf(held[j][x], held[j][x], ss);
    }
    for (int c = V * (lane + LANES * HELD); c < part; c += V * LANES) {
        const vec u = *reinterpret_cast<const vec*>(yr + c) * inv_size;
#pragma unroll
        for (int x = 0; x < V; ++x) ss = fmaf(u[x], u[x], ss);
    }
    ss = LANES == 256 ? block_sum<256>(ss, red) : wave_sum(ss);
    const float inv = scale / sqrtf(ss / (float)part + eps);
    T* to = out + t * out_stride + at;
    auto store = [&](int c, vec u) {
        const vec gate = *reinterpret_cast<const vec*>(gr + c), ww = *reinterpret_cast<const vec*>(w + at + c);
        tvec o;
#pragma unroll
        for (int x = 0; x < V; ++x) o[x] = from_float<T>(u[x] * inv * ww[x] / (1.0f + expf(-gate[x])));
        *reinterpret_cast<tvec*>(to + c) = o;
    };
#pragma unroll
    for (int j = 0; j < HELD; ++j) {
        const int c = V * (lane + LANES * j);
        if (c < part) store(c, held[j]);
    }
    for (int c = V * (lane + LANES * HELD); c < part; c += V * LANES) store(c, *reinterpret_cast<const vec*>(yr + c) * inv_size);
}

extern "C" int somi_norm_sigmoid_gate(const float* y, const float* den, const float* floor_, const float* g, int64_t g_stride,
                                      const float* w, int groups, float eps, float scale, int n_tokens, int width, void* out,
                                      int64_t out_stride, int dtype, hipStream_t stream) {
    SOMI_REQUIRE(n_tokens >= 0 && width > 0 && groups > 0 && width % groups == 0, "norm_sigmoid_gate: %d values in %d parts", width, groups);
    SOMI_REQUIRE(g_stride >= width && out_stride >= width, "norm_sigmoid_gate: bad strides");
    SOMI_REQUIRE((den == nullptr) == (floor_ == nullptr), "norm_sigmoid_gate: a normaliser comes with its floor");
    SOMI_REQUIRE(dtype == SOMI_F32 || dtype == SOMI_BF16, "norm_sigmoid_gate: unknown dtype %d", dtype);
    if (n_tokens == 0) return 0;
    const int part = width / groups;
    const int64_t units = (int64_t)n_tokens * groups;
    const bool vec = part % 4 == 0 && g_stride % 4 == 0 && out_stride % 4 == 0 && (uintptr_t)y % 16 == 0 && (uintptr_t)g % 16 == 0 &&
                     (uintptr_t)w % 16 == 0 && (uintptr_t)out % 16 == 0;
    const bool wave = part <= 1024;                          // a wavefront a part, four of them a workgroup
    const int64_t blocks = wave ? ceil_div64(units, 4) : units;
    SOMI_REQUIRE(blocks <= 0x7fffffff, "norm_sigmoid_gate: too many rows");
#define SOMI_NSG(T, L, V)                                                                                                    \
    hipLaunchKernelGGL((norm_sigmoid_gate_kernel<T, L, V>), dim3((unsigned)blocks), dim3(256), 0, stream, y, den, floor_, g, \
                       g_stride, w, eps, scale, groups, width, part, units, (T*)out, out_stride)
#define SOMI_NSG_AS(T)                                        \
    do {                                                      \
        if (wave && vec) SOMI_NSG(T, 64, 4);                  \
        else if (wave) SOMI_NSG(T, 64, 1);                    \
        else if (vec) SOMI_NSG(T, 256, 4);                    \
        else SOMI_NSG(T, 256, 1);                             \
    } while (0)
    if (dtype == SOMI_F32) SOMI_NSG_AS(float);
    else SOMI_NSG_AS(bf16);
#undef SOMI_NSG_AS
#undef SOMI_NSG
    SOMI_LAUNCH_CHECK("norm_sigmoid_gate");
    return 0;
}
