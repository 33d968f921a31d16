// The linear recurrence with ONE constant decay g a head over chunks of tokens on the matrix cores (bfloat16 engine, the
// many rows of prompt portions):
//     S_t = g S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t        (S: N key channels x V value channels, 32-bit).
// A request's rows of the step are cut into chunks of at most `chunk` tokens (a multiple of 64), numbered t = 0 .. n - 1
// within a chunk; with S0 the state a chunk starts from,
//     o_t = g^(t+1) S0^T q_t + sum_(s<=t) g^(t-s) (q_t . k_s) v_s,      S1 = g^n S0 + sum_s g^(n-1-s) k_s v_s^T.
// Three launches: what every chunk adds to its state (the last sum), all chunks side by side; the states the chunks start
// from, a request's chunks in their order, element by element (and the state after the step, staged); every chunk's
// outputs, 64 rows a workgroup.
//
// 32-bit operands on matrix cores that multiply bfloat16: an operand is the sum of three bfloat16 numbers of 8 significant
// bits each, which holds a 32-bit number's 24 bits whole; a product is the six (or three, where the other operand is
// bfloat16 as it comes) products of parts whose orders add up to less than three, summed in 32-bit: what is left out lies
// below 2^-22 of the product.  Decays, activations and rotations are 32-bit too.
#define MLR_BF16 1
#include "common.h"

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;
typedef __attribute__((__vector_size__(4 * sizeof(uint32_t)))) uint32_t u32x4;

#define BT 64                // tokens of a block: the rows of an output workgroup, and what is staged at a time
#define TP (BT + 8)          // elements between the channels of a transposed block
#define VB 128               // value channels of a workgroup
#define PARTS 3
#define THREADS 512
#define MAX_CHUNK_KEYS 128

struct ChunkArgs {
    const __bf16* q; long q_stride;            // q[r * q_stride + (head / heads_per_group) * N + i], as projected
    const __bf16* k; long k_stride;
    const __bf16* v; long v_stride;            // v[r * v_stride + head * V + j]
    const float* log_decay;                    // [heads]
    float* out;                                // [rows, heads * V]
    const float* live; float* stage; long state_stride;     // a request's S as [heads][N][V]
    const int32_t* slots;
    const int32_t* seg_first; const int32_t* seg_count;     // the step's requests
    const int32_t* chunk_first; const int32_t* chunk_count; // their chunks, a request's one after the other
    float* chunk_state;                        // [chunks][heads][V][N]: what a chunk adds, then what it starts from
    const float* rope; const int32_t* positions;
    int rot_dim, chunk, heads, heads_per_group, N, V, write_state, silu;
    float q_scale;
};

#define LOG2E 1.4426950408889634f
// (the exponential and reciprocal instructions: 32-bit, each within a unit of the last place or so)
__device__ __forceinline__ float silu_of(float x) { return x * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-LOG2E * x)); }

// Eight channels of a row from channel `ch` on, through the activation and the rotation (pairs (i, i + rot_dim / 2)).
__device__ __forceinline__ void row_channels(const ChunkArgs& a, const __bf16* head_row, size_t row, int ch, float (&x)[8]) {
    load_vec(head_row + ch, x);
    if (a.silu)
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = silu_of(x[e]);
    if (ch < a.rot_dim) {
        const int half = a.rot_dim >> 1;
        const bool low = ch < half;
        const int j = low ? ch : ch - half;
        float o[8], c[8], s[8];
        load_vec(head_row + (low ? ch + half : ch - half), o);
        const float* cs = a.rope + (size_t)a.positions[row] * a.rot_dim + j;
#pragma unroll
        for (int e = 0; e < 8; e += 4) {
            *reinterpret_cast<float4*>(c + e) = *reinterpret_cast<const float4*>(cs + e);
            *reinterpret_cast<float4*>(s + e) = *reinterpret_cast<const float4*>(cs + half + e);
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float other = a.silu ? silu_of(o[e]) : o[e];
            x[e] = low ? turn_x(x[e], other, c[e], s[e]) : turn_y(other, x[e], c[e], s[e]);
        }
    }
}

// x as a sum of bfloat16 numbers: a part is the upper half of what the parts before it leave (cut off, so each holds the
// next eight significant bits); P 1: x holds bfloat16 numbers.
template <int P> __device__ __forceinline__ void parts_of(const float (&x)[8], bf16x8 (&part)[P]) {
    u32x4 w[P];
#pragma unroll
    for (int c = 0; c < 4; ++c) {
        float lo = x[2 * c], hi = x[2 * c + 1];
#pragma unroll
        for (int p = 0; p < P; ++p) {
            const uint32_t a = __float_as_uint(lo), b = __float_as_uint(hi);
            w[p][c] = __builtin_amdgcn_perm(b, a, 0x07060302u);          // the upper halves of both
            if (p + 1 < P) {
                lo -= __uint_as_float(a & 0xffff0000u);
                hi -= __uint_as_float(b & 0xffff0000u);
            }
        }
    }
#pragma unroll
    for (int p = 0; p < P; ++p) part[p] = __builtin_bit_cast(bf16x8, w[p]);
}

// Eight channels of one token into [part][channel][TP]: the lane beside holds the token beside, so a lane takes the other's
// halves by a lane exchange and writes the pair (token, token + 1) of a channel as one word.
template <int P> __device__ __forceinline__ void put_transposed(__bf16* dst, int channels, int ch, int token, const float (&x)[8]) {
    bf16x8 part[P];
    parts_of<P>(x, part);
    const bool odd = token & 1;
#pragma unroll
    for (int p = 0; p < P; ++p) {
        const u32x4 w = __builtin_bit_cast(u32x4, part[p]);
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            const uint32_t own = w[c];
            const uint32_t other = (uint32_t)__builtin_amdgcn_mov_dpp((int)own, 0xB1, 0xF, 0xF, true);   // lane ^ 1
            const uint32_t pair = odd ? ((other >> 16) | (own & 0xffff0000u)) : ((own & 0xffffu) | (other << 16));
            *reinterpret_cast<uint32_t*>(&dst[((size_t)p * channels + ch + 2 * c + (odd ? 1 : 0)) * TP + (token & ~1)]) = pair;
        }
    }
}

// acc += the product of two 32-bit operands given in parts
template <int PA, int PB> __device__ __forceinline__ void multiply(floatx4& acc, const bf16x8 (&x)[PA], const bf16x8 (&y)[PB]) {
#pragma unroll
    for (int i = 0; i < PA; ++i)
#pragma unroll
        for (int j = 0; j < PB; ++j)
            if (i + j < PARTS) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x[i], y[j], acc, 0, 0, 0);
}

template <int P> __device__ __forceinline__ void fragment(bf16x8 (&f)[P], const __bf16* src, size_t part_stride) {
#pragma unroll
    for (int p = 0; p < P; ++p) f[p] = *reinterpret_cast<const bf16x8*>(src + p * part_stride);
}

// chunk_state[chunk][head][v][n] = sum_s g^(n_tokens - 1 - s) k_s[n] v_s[v]: one workgroup a chunk, head and VB value
// channels.  A wavefront owns 16 key channels (where they are fewer than eight times 16, several share one and deal the
// value channels out).  VP: parts of a value (1: bfloat16 as it comes).
template <int VP>
__global__ __launch_bounds__(THREADS) void chunk_write_kernel(ChunkArgs a) {
    extern __shared__ __attribute__((aligned(16))) unsigned char lds_raw[];
    const int N = a.N, V = a.V, nt = (N + 15) >> 4, n_rows = nt * 16;
    __bf16* k_t = reinterpret_cast<__bf16*>(lds_raw);                 // [PARTS][n_rows][TP]
    __bf16* v_t = k_t + (size_t)PARTS * n_rows * TP;                   // [VP][VB][TP]
    const int chunk = blockIdx.x, head = blockIdx.y, v0 = blockIdx.z * VB;
    const int first = a.chunk_first[chunk], count = a.chunk_count[chunk];
    const int v_cols = min(VB, V - v0), vt = v_cols >> 4;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, i16 = lane & 15, b = lane >> 4;
    const float lam = a.log_decay[head] * LOG2E;
    const int shares = 8 / nt, my_nt = wave % nt, share = wave / nt;
    floatx4 acc[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[j] = floatx4{0.f, 0.f, 0.f, 0.f};
    for (int t0 = 0; t0 < count; t0 += BT) {
        __syncthreads();                                                // (the block before has been read)
        for (int i = tid; i < BT * (n_rows >> 3); i += THREADS) {       // (whole wavefronts: 64 tokens of eight channels)
            const int token = i & 63, ch = (i >> 6) * 8;
            float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            if (t0 + token < count && ch < N) {
                const size_t row = (size_t)(first + t0 + token);
                row_channels(a, a.k + row * a.k_stride + (head / a.heads_per_group) * N, row, ch, x);
                const float f = __builtin_amdgcn_exp2f(lam * (float)(count - 1 - t0 - token));
#pragma unroll
                for (int e = 0; e < 8; ++e) x[e] *= f;
            }
            put_transposed<PARTS>(k_t, n_rows, ch, token, x);
        }
        for (int i = tid; i < BT * (v_cols >> 3); i += THREADS) {
            const int token = i & 63, ch = (i >> 6) * 8;
            float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            if (t0 + token < count) {
                load_vec(a.v + (size_t)(first + t0 + token) * a.v_stride + (size_t)head * V + v0 + ch, x);
                if (VP > 1)
#pragma unroll
                    for (int e = 0; e < 8; ++e) x[e] = silu_of(x[e]);
            }
            put_transposed<VP>(v_t, VB, ch, token, x);
        }
        __syncthreads();
        if (share < shares) {
#pragma unroll
            for (int ks = 0; ks < BT; ks += 32) {
                bf16x8 kf[PARTS];
                fragment<PARTS>(kf, k_t + (my_nt * 16 + i16) * TP + ks + 8 * b, (size_t)n_rows * TP);
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    const int tile = share + shares * j;
                    if (tile < vt) {                                     // (the same in every lane)
                        bf16x8 vf[VP];
                        fragment<VP>(vf, v_t + (tile * 16 + i16) * TP + ks + 8 * b, (size_t)VB * TP);
                        multiply<PARTS, VP>(acc[j], kf, vf);
                    }
                }
            }
        }
    }
    if (share >= shares) return;
    float* dst = a.chunk_state + ((size_t)chunk * a.heads + head) * N * V;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        const int tile = share + shares * j, n = my_nt * 16 + 4 * b;     // accumulator element r: key channel n + r, value channel i16
        if (tile < vt && n < N)
            *reinterpret_cast<float4*>(dst + (size_t)(v0 + tile * 16 + i16) * N + n) = make_float4(acc[j][0], acc[j][1], acc[j][2], acc[j][3]);
    }
}

// The states the chunks start from: one thread per (request, head, value channel, key channel) walks the request's chunks.
#define STATE_AHEAD 4
__global__ __launch_bounds__(256) void chunk_states_kernel(ChunkArgs a) {
    const int n = blockIdx.x * 64 + (threadIdx.x & 63), v = blockIdx.y * 4 + (threadIdx.x >> 6);
    const int seg = blockIdx.z / a.heads, head = blockIdx.z % a.heads;
    int chunk0 = 0;
    for (int s = 0; s < seg; ++s) chunk0 += (a.seg_count[s] + a.chunk - 1) / a.chunk;
    const int chunks = (a.seg_count[seg] + a.chunk - 1) / a.chunk, slot = a.slots[a.seg_first[seg]];
    if (n >= a.N || v >= a.V) return;
    const size_t at = (size_t)slot * a.state_stride + ((size_t)head * a.N + n) * a.V + v;
    const size_t per = (size_t)a.heads * a.N * a.V;
    float* p = a.chunk_state + (size_t)chunk0 * per + ((size_t)head * a.V + v) * a.N + n;
    const float lam = a.log_decay[head] * LOG2E;
    float S = a.live[at];
    for (int c0 = 0; c0 < chunks; c0 += STATE_AHEAD) {
        float add[STATE_AHEAD];
#pragma unroll
        for (int i = 0; i < STATE_AHEAD; ++i) add[i] = c0 + i < chunks ? p[(size_t)(c0 + i) * per] : 0.f;
#pragma unroll
        for (int i = 0; i < STATE_AHEAD; ++i) {
            if (c0 + i < chunks) {
                p[(size_t)(c0 + i) * per] = S;
                S = __builtin_amdgcn_exp2f(lam * (float)a.chunk_count[chunk0 + c0 + i]) * S + add[i];
            }
        }
    }
    if (a.write_state) a.stage[at] = S;
}

// Outputs: one workgroup per 64 rows of a chunk, head and VB value channels.  The rows' queries lie in LDS; the state's
// part first (a wavefront owns 16 value channels: it reads its rows of the state once, straight from memory), then for
// every block of 64 keys up to the rows' own: scores (keys x rows, so that a lane holds eight neighbouring keys of one row),
// decayed and written to LDS in parts, and their product with the block's values.
template <int VP>
__global__ __launch_bounds__(THREADS) void chunk_read_kernel(ChunkArgs a, int blocks_a_chunk) {
    extern __shared__ __attribute__((aligned(16))) unsigned char lds_raw[];
    const int N = a.N, V = a.V, n_steps = (N + 31) >> 5, pitch = n_steps * 32 + 8;
    __bf16* q_l = reinterpret_cast<__bf16*>(lds_raw);                  // [PARTS][BT][pitch]
    __bf16* p_l = q_l + (size_t)PARTS * BT * pitch;                     // [PARTS][BT][TP]
    __bf16* k_l = p_l + (size_t)PARTS * BT * TP;                        // [PARTS][BT][pitch], and in its place
    __bf16* v_t = k_l;                                                   // [VP][VB][TP]
    const int chunk = blockIdx.x / blocks_a_chunk, block = blockIdx.x % blocks_a_chunk, head = blockIdx.y, v0 = blockIdx.z * VB;
    const int first = a.chunk_first[chunk], count = a.chunk_count[chunk];
    if (block * BT >= count) return;
    const int rows = min(BT, count - block * BT);
    const int v_cols = min(VB, V - v0), vt = v_cols >> 4;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, i16 = lane & 15, b = lane >> 4;
    const float lam = a.log_decay[head] * LOG2E;
    const int qk_head = head / a.heads_per_group;
    // this wavefront's value channels and rows: with few value channels several wavefronts share 16 of them and deal the rows out
    const int shares = vt > 4 ? 1 : vt > 2 ? 2 : 4, my_vt = wave / shares, share = wave % shares, tiles = 4 / shares;
    const bool mine = my_vt < vt;
    float s0[4][8];
    if (mine) {
        const float* src = a.chunk_state + (((size_t)chunk * a.heads + head) * V + v0 + my_vt * 16 + i16) * N;
#pragma unroll
        for (int ks = 0; ks < 4; ++ks) {
            const int n = ks * 32 + 8 * b;
            const float4 lo = n < N ? *reinterpret_cast<const float4*>(src + n) : make_float4(0.f, 0.f, 0.f, 0.f);
            const float4 hi = n < N ? *reinterpret_cast<const float4*>(src + n + 4) : make_float4(0.f, 0.f, 0.f, 0.f);
            s0[ks][0] = lo.x; s0[ks][1] = lo.y; s0[ks][2] = lo.z; s0[ks][3] = lo.w;
            s0[ks][4] = hi.x; s0[ks][5] = hi.y; s0[ks][6] = hi.z; s0[ks][7] = hi.w;
        }
    }
    // 64 rows of q or k into [part][row][pitch], zeros past the rows there are and past the key channels
    auto put_rows = [&](const __bf16* base, long stride, int row0, int present, float factor, __bf16* dst) {
        for (int i = tid; i < BT * (MAX_CHUNK_KEYS / 8); i += THREADS) {
            const int r = i / (MAX_CHUNK_KEYS / 8), ch = (i % (MAX_CHUNK_KEYS / 8)) * 8;
            if (ch >= n_steps * 32) continue;
            float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            if (r < present && ch < N) {
                const size_t row = (size_t)(row0 + r);
                row_channels(a, base + row * stride + qk_head * N, row, ch, x);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[e] *= factor;
            }
            bf16x8 part[PARTS];
            parts_of<PARTS>(x, part);
#pragma unroll
            for (int p = 0; p < PARTS; ++p) *reinterpret_cast<bf16x8*>(&dst[((size_t)p * BT + r) * pitch + ch]) = part[p];
        }
    };
    put_rows(a.q, a.q_stride, first + block * BT, rows, a.q_scale, q_l);
    put_rows(a.k, a.k_stride, first, min(BT, count), 1.0f, k_l);
    __syncthreads();
    floatx4 acc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = floatx4{0.f, 0.f, 0.f, 0.f};
    if (mine) {
#pragma unroll
        for (int ks = 0; ks < 4; ++ks) {
            if (ks < n_steps) {
                bf16x8 sf[PARTS];
                parts_of<PARTS>(s0[ks], sf);
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    if (j < tiles) {
                        bf16x8 qf[PARTS];
                        fragment<PARTS>(qf, q_l + ((share + shares * j) * 16 + i16) * pitch + ks * 32 + 8 * b, (size_t)BT * pitch);
                        multiply<PARTS, PARTS>(acc[j], sf, qf);
                    }
                }
            }
        }
#pragma unroll
        for (int j = 0; j < 4; ++j)
            if (j < tiles) acc[j] *= __builtin_amdgcn_exp2f(lam * (float)(block * BT + (share + shares * j) * 16 + i16 + 1));
    }
    const int row_tile = wave & 3, key_half = wave >> 2;                 // of the scores
    const int key_row = key_half * 32 + 8 * (i16 >> 2) + (i16 & 3);      // (and key_row + 4)
    for (int kb = 0; kb <= block; ++kb) {
        const int keys = min(BT, count - kb * BT);
        if (kb > 0) {
            __syncthreads();                                              // (the block before has been read)
            put_rows(a.k, a.k_stride, first + kb * BT, keys, 1.0f, k_l);
            __syncthreads();
        }
        // the block's values are on their way while the scores are taken
        float vx[VB * BT / 8 / THREADS][8];
#pragma unroll
        for (int u = 0; u < VB * BT / 8 / THREADS; ++u) {
            const int i = tid + u * THREADS, token = i & 63, ch = (i >> 6) * 8;
#pragma unroll
            for (int e = 0; e < 8; ++e) vx[u][e] = 0.f;
            if (token < keys && ch < v_cols)
                load_vec(a.v + (size_t)(first + kb * BT + token) * a.v_stride + (size_t)head * V + v0 + ch, vx[u]);
        }
        floatx4 s_lo = {0.f, 0.f, 0.f, 0.f}, s_hi = {0.f, 0.f, 0.f, 0.f};
        if (kb < block || key_half * 32 <= row_tile * 16 + 15) {          // (else every key lies behind every row)
            for (int ks = 0; ks < n_steps; ++ks) {
                bf16x8 qf[PARTS], kf[PARTS];
                fragment<PARTS>(qf, q_l + (row_tile * 16 + i16) * pitch + ks * 32 + 8 * b, (size_t)BT * pitch);
                fragment<PARTS>(kf, k_l + key_row * pitch + ks * 32 + 8 * b, (size_t)BT * pitch);
                multiply<PARTS, PARTS>(s_lo, kf, qf);
                fragment<PARTS>(kf, k_l + (key_row + 4) * pitch + ks * 32 + 8 * b, (size_t)BT * pitch);
                multiply<PARTS, PARTS>(s_hi, kf, qf);
            }
        }
        {
            const int t = row_tile * 16 + i16, behind = (block - kb) * BT + t - key_half * 32 - 8 * b;   // row minus the lane's first key
            float w[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float s = e < 4 ? s_lo[e] : s_hi[e - 4];
                w[e] = behind - e >= 0 ? s * __builtin_amdgcn_exp2f(lam * (float)(behind - e)) : 0.f;
            }
            bf16x8 part[PARTS];
            parts_of<PARTS>(w, part);
#pragma unroll
            for (int p = 0; p < PARTS; ++p) *reinterpret_cast<bf16x8*>(&p_l[((size_t)p * BT + t) * TP + key_half * 32 + 8 * b]) = part[p];
        }
        __syncthreads();                                                  // (the keys have been read: the values take their place)
#pragma unroll
        for (int u = 0; u < VB * BT / 8 / THREADS; ++u) {
            const int i = tid + u * THREADS, token = i & 63, ch = (i >> 6) * 8;
            if (VP > 1)
#pragma unroll
                for (int e = 0; e < 8; ++e) vx[u][e] = silu_of(vx[u][e]);
            if (ch < v_cols) put_transposed<VP>(v_t, VB, ch, token, vx[u]);      // (the same in every lane)
        }
        __syncthreads();
        if (mine) {
#pragma unroll
            for (int ks = 0; ks < BT; ks += 32) {
                bf16x8 vf[VP];
                fragment<VP>(vf, v_t + (my_vt * 16 + i16) * TP + ks + 8 * b, (size_t)VB * TP);
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    if (j < tiles) {
                        bf16x8 pf[PARTS];
                        fragment<PARTS>(pf, p_l + ((share + shares * j) * 16 + i16) * TP + ks + 8 * b, (size_t)BT * TP);
                        multiply<VP, PARTS>(acc[j], vf, pf);
                    }
                }
            }
        }
    }
    if (!mine) return;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int t = (share + shares * j) * 16 + i16;                    // accumulator element r: value channel 4 b + r of row t
        if (j < tiles && t < rows)
            *reinterpret_cast<float4*>(a.out + (size_t)(first + block * BT + t) * ((size_t)a.heads * V) + (size_t)head * V + v0 + my_vt * 16 + 4 * b) =
                make_float4(acc[j][0], acc[j][1], acc[j][2], acc[j][3]);
    }
}

template <class Kernel> static int raise_lds(Kernel* kernel, size_t bytes, bool& raised) {
    if (raised || bytes <= 48 * 1024) return 0;
    if (hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) != hipSuccess) return -3;
    raised = true;
    return 0;
}

template <int VP> static int launch_chunks(const ChunkArgs& a, int segments, int chunks, hipStream_t stream) {
    static bool raised_write = false, raised_read = false;
    const int n_rows = (a.N + 15) / 16 * 16, pitch = (a.N + 31) / 32 * 32 + 8, v_blocks = (a.V + VB - 1) / VB;
    const size_t lds_write = sizeof(__bf16) * ((size_t)PARTS * n_rows * TP + (size_t)VP * VB * TP);
    const size_t keys = (size_t)PARTS * BT * pitch, values = (size_t)VP * VB * TP;
    const size_t lds_read = sizeof(__bf16) * ((size_t)PARTS * BT * pitch + (size_t)PARTS * BT * TP + (keys > values ? keys : values));
    int err = raise_lds(&chunk_write_kernel<VP>, lds_write, raised_write);
    if (err != 0) return err;
    err = raise_lds(&chunk_read_kernel<VP>, lds_read, raised_read);
    if (err != 0) return err;
    chunk_write_kernel<VP><<<dim3(chunks, a.heads, v_blocks), THREADS, lds_write, stream>>>(a);
    err = (int)hipGetLastError();
    if (err != 0) return err;
    chunk_states_kernel<<<dim3((a.N + 63) / 64, (a.V + 3) / 4, (unsigned)segments * a.heads), 256, 0, stream>>>(a);
    err = (int)hipGetLastError();
    if (err != 0) return err;
    const int blocks = a.chunk / BT;
    chunk_read_kernel<VP><<<dim3((unsigned)chunks * blocks, a.heads, v_blocks), THREADS, lds_read, stream>>>(a, blocks);
    return (int)hipGetLastError();
}

extern "C" {

// `seg_first`/`seg_count`: the step's requests (first row, rows); `chunk_first`/`chunk_count`: their chunks of at most
// `chunk` tokens, a request's one after the other and the requests in the same order.  chunk_state: chunks * heads *
// n_keys * n_values floats.  Up to 128 key channels a head in multiples of 8, value channels in multiples of 16, rows and
// heads that start at multiples of 16 bytes, a rotation whose halves are multiples of 8 channels.
int mlr_decayed_recurrence_chunks(const void* q, long q_stride, const void* k, long k_stride, const void* v, long v_stride,
                                  const float* log_decay, float q_scale, int silu, const float* rope, const int32_t* positions,
                                  int rot_dim, float* out, const float* live, float* stage, long state_stride, const int32_t* slots,
                                  const int32_t* seg_first, const int32_t* seg_count, int segments, const int32_t* chunk_first,
                                  const int32_t* chunk_count, int chunks, int chunk, float* chunk_state, int heads,
                                  int heads_per_group, int n_keys, int n_values, int write_state, hipStream_t stream) {
    if (segments <= 0 || chunks <= 0) return 0;
    const auto aligned = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
    if (n_keys < 8 || n_keys > MAX_CHUNK_KEYS || n_keys % 8 != 0 || n_values < 16 || n_values % 16 != 0 || heads < 1 ||
        heads_per_group < 1 || heads % heads_per_group != 0 || heads > 65535 || (long)segments * heads > 65535 || chunk < BT ||
        chunk % BT != 0 || rot_dim < 0 || rot_dim > n_keys || rot_dim % 16 != 0 ||
        (rot_dim > 0 && (rope == nullptr || positions == nullptr || !aligned(rope))) || q_stride % 8 != 0 || k_stride % 8 != 0 ||
        v_stride % 8 != 0 || !aligned(q) || !aligned(k) || !aligned(v) || !aligned(out) || !aligned(chunk_state) || (n_values + 3) / 4 > 65535)
        return -1;
    ChunkArgs a{(const __bf16*)q, q_stride, (const __bf16*)k, k_stride, (const __bf16*)v, v_stride, log_decay, out, live, stage,
                state_stride, slots, seg_first, seg_count, chunk_first, chunk_count, chunk_state, rope, positions, rot_dim, chunk,
                heads, heads_per_group, n_keys, n_values, write_state, silu, q_scale};
    return silu ? launch_chunks<3>(a, segments, chunks, stream) : launch_chunks<1>(a, segments, chunks, stream);
}

int mlr_decayed_chunk_block() { return BT; }

}  // extern "C"
