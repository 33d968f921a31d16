// Causal softmax attention over the paged cache whose heads are mixed between the softmax and the values:
//   s_h(i, j)  = (q_h(i) . k_kv(h)(j)) * scale, then softcap * tanh(s / softcap) when softcap > 0
//   p_h(i, j)  = exp(s_h) / (sum_j exp(s_h) + exp(sink))       (sink: a constant, a number a head, or none)
//   w_h(i, j)  = sum_g mix[h, g] p_g(i, j)
//   o_h(i)     = sum_j w_h(i, j) v_kv(h)(j)
// and whose values may be turned by their position before they are cached: o_h(i) is then turned back by the
// query's own position, and at last multiplied by one gate a head, sigmoid(gate[i, h]).  kv(h) = h / (q_heads /
// kv_heads).  Scores, softmax, sums, the turn and the gate are 32-bit.
//
// Cache of one layer: keys k_pages[page][kv_head][place in page][key_dim], values transposed within a page,
// v_pages[page][kv_head][value_dim][place].
//
// `head_mix_attention_kernel`: one workgroup a token, any sizes, both engines; tiles of 64 keys at absolute multiples
// of 64, so a token's sums and their order follow from its own position alone.
//
// On the matrix cores (bfloat16), three launches over groups of up to NQ consecutive tokens of a request:
//   `head_scores_kernel`   e = exp(s) of every (token, key, head) into scratch, and the sums of e;
//   `head_mix_values_kernel`  weights e / sum, mixed over the heads by one product with `mix`, times the values;
//   `head_mix_finish_kernel`  the shares of the key ranges added, turned back, gated.
// A mixed weight needs the finished sums of ALL heads, so the weights cannot be mixed on the first walk over the keys
// (a walk that keeps every head's sums over every kv head's values instead does kv_heads times the work of the second
// product).  Scores are bounded by the cap, so exp(s) is taken without a running maximum (caps up to 60: exp(60) times
// 2^24 keys fits 32 bits) and nothing is ever rescaled.
#include "common.h"

struct HeadMixArgs {
    const elem_t* q; long q_stride;            // q[m * q_stride + head * key_dim + d]
    const elem_t* k_pages; const elem_t* v_pages;
    const int32_t* block_table; const int32_t* slots; const int32_t* positions;
    const float* mix;                          // [q_heads, q_heads]
    const float* sink; float sink_value; int sink_kind;      // 0: none, 1: sink_value for every head, 2: sink[head]
    const float* v_rope; int v_interleaved;    // [positions, value_dim]: cosines | sines of value_dim / 2 pairs; null: not turned
    const elem_t* gate; long gate_stride;      // gate[m * gate_stride + head] or null
    elem_t* out; long out_stride;              // out[m * out_stride + head * value_dim + c]
    int max_blocks, q_heads, kv_heads, key_dim, value_dim, page_size;
    float scale, softcap;
};

// Channel c of a head's output x (value_dim channels, `at(i)` gives one) turned back by position `pos`.
template <class At>
__device__ __forceinline__ float turned_back(const At& at, int c, const float* cs, int dim, int interleaved) {
    if (cs == nullptr) return at(c);
    const int half = dim >> 1;
    const int j = interleaved ? c >> 1 : (c < half ? c : c - half);
    const bool low = interleaved ? !(c & 1) : c < half;
    const float co = cs[j], si = cs[half + j];
    const float u = at(interleaved ? 2 * j : j), v = at(interleaved ? 2 * j + 1 : j + half);
    return low ? turn_x(u, v, co, -si) : turn_y(u, v, co, -si);
}

__device__ __forceinline__ float sink_term(const HeadMixArgs& a, int head) {
    return a.sink_kind == 1 ? a.sink_value : a.sink_kind == 2 ? a.sink[head] : -INFINITY;
}

#define TILE_KEYS 64

// LDS: p[q_heads][64], w[q_heads][64], acc[q_heads * value_dim], top[q_heads], inv[q_heads] floats.
__global__ __launch_bounds__(256) void head_mix_attention_kernel(HeadMixArgs a) {
    extern __shared__ float lds[];
    __shared__ long long k_at[TILE_KEYS];      // element offsets of a key's row / of its column of values, kv head 0
    __shared__ long long v_at[TILE_KEYS];
    const int H = a.q_heads, D = a.key_dim, V = a.value_dim, PS = a.page_size;
    float* p = lds;
    float* w = p + H * TILE_KEYS;
    float* acc = w + H * TILE_KEYS;
    float* top = acc + (size_t)H * V;
    float* inv = top + H;
    const int m = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int hg = H / a.kv_heads;
    const int pos = a.positions[m];
    const int32_t* table = a.block_table + (size_t)a.slots[m] * a.max_blocks;
    for (int i = tid; i < H * V; i += 256) acc[i] = 0.f;
    for (int h = tid; h < H; h += 256) {
        top[h] = -INFINITY;
        inv[h] = 0.f;
    }
    auto place = [&](int t0) {                 // (between barriers)
        if (tid < TILE_KEYS) {
            const int kp = t0 + tid, block = kp / PS;
            const int page = (kp <= pos && block < a.max_blocks) ? table[block] : -1;
            k_at[tid] = page >= 0 ? ((long long)page * a.kv_heads * PS + kp % PS) * D : -1;
            v_at[tid] = page >= 0 ? (long long)page * a.kv_heads * V * PS + kp % PS : -1;
        }
    };
    auto score = [&](int h) {                  // of this lane's key; -inf where it is not seen
        const long long at = k_at[lane];
        if (at < 0) return -INFINITY;
        const elem_t* kr = a.k_pages + at + (long long)(h / hg) * PS * D;
        const elem_t* qr = a.q + (size_t)m * a.q_stride + (size_t)h * D;
        float s = 0.f;
        for (int d = 0; d < D; ++d) s = fmaf(to_float(qr[d]), to_float(kr[d]), s);
        s *= a.scale;
        return a.softcap > 0.f ? a.softcap * tanhf(s / a.softcap) : s;
    };
    // first walk: every head's maximum and sum (a wavefront a head)
    for (int t0 = 0; t0 <= pos; t0 += TILE_KEYS) {
        __syncthreads();
        place(t0);
        __syncthreads();
        for (int h = wave; h < H; h += 4) {
            const float s = score(h);
            const float old = top[h], now = fmaxf(old, wave_max(s));
            const float e = s > -INFINITY ? expf(s - now) : 0.f;
            const float sum = (old > -INFINITY ? inv[h] * expf(old - now) : 0.f) + wave_sum(e);
            if (lane == 0) {
                top[h] = now;
                inv[h] = sum;
            }
        }
    }
    __syncthreads();
    for (int h = tid; h < H; h += 256) {
        const float sk = sink_term(a, h), now = fmaxf(top[h], sk);
        const float den = (top[h] > -INFINITY ? inv[h] * expf(top[h] - now) : 0.f) + (sk > -INFINITY ? expf(sk - now) : 0.f);
        top[h] = now;
        inv[h] = den > 0.f ? 1.0f / den : 0.f;
    }
    // second walk: the weights, mixed, times the values
    for (int t0 = 0; t0 <= pos; t0 += TILE_KEYS) {
        __syncthreads();
        place(t0);
        __syncthreads();
        for (int h = wave; h < H; h += 4) {
            const float s = score(h);
            p[h * TILE_KEYS + lane] = s > -INFINITY ? expf(s - top[h]) * inv[h] : 0.f;
        }
        __syncthreads();
        for (int h = wave; h < H; h += 4) {
            float sum = 0.f;
            for (int g = 0; g < H; ++g) sum = fmaf(a.mix[(size_t)h * H + g], p[g * TILE_KEYS + lane], sum);
            w[h * TILE_KEYS + lane] = sum;
        }
        __syncthreads();
        const int keys = min(TILE_KEYS, pos + 1 - t0);
        for (int o = tid; o < H * V; o += 256) {
            const int h = o / V, c = o % V;
            const elem_t* vr = a.v_pages + ((long long)(h / hg) * V + c) * PS;
            float sum = acc[o];
            for (int key = 0; key < keys; ++key)
                if (v_at[key] >= 0) sum = fmaf(w[h * TILE_KEYS + key], to_float(vr[v_at[key]]), sum);
            acc[o] = sum;
        }
    }
    __syncthreads();
    const float* cs = a.v_rope ? a.v_rope + (size_t)pos * V : nullptr;
    for (int o = tid; o < H * V; o += 256) {
        const int h = o / V, c = o % V;
        const float* row = acc + (size_t)h * V;
        float y = turned_back([&](int i) { return row[i]; }, c, cs, V, a.v_interleaved);
        if (a.gate != nullptr) y *= 1.0f / (1.0f + expf(-to_float(a.gate[(size_t)m * a.gate_stride + h])));
        a.out[(size_t)m * a.out_stride + o] = from_float<elem_t>(y);
    }
}

#if MLR_BF16
// ---------------------------------------------------------------------------------------------------------
// The matrix-core form.  Heads are numbered in a padded order: the q_heads / kv_heads heads of a kv head take `hp` (a
// power of two) places, index = kv * hp + head within it, and kv heads are padded to `kv_pad` = head_k / hp, head_k
// being 16 or a multiple of 32 (the inner size of the product that mixes the heads); padding holds zeros.
//
// Scratch of a (token row, tile of 32 keys, half s, step of heads): the 64 lanes' operands of that product as they
// lie -- lane (b, i) has the consecutive heads of key 8 (i / 4) + 4 s + i % 4: a load is one coalesced access a
// wavefront.  The order of the keys makes the product leave eight CONSECUTIVE keys of one head in a lane (four from
// each half), which is the operand of the product with the values.
typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(__bf16)))) __bf16 bf16x4;
typedef __attribute__((__vector_size__(2 * sizeof(__bf16)))) __bf16 bf16x2;
typedef __attribute__((__vector_size__(4 * sizeof(short)))) short shortx4;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;

#define TK 32                   // keys in a tile

// The product that mixes the heads: four heads a lane (inner size 16) or eight (32).
__device__ __forceinline__ floatx4 mixed(bf16x4 p, bf16x8 m, floatx4 d) {
    const bf16x4 m4 = {m[0], m[1], m[2], m[3]};
    return __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(__builtin_bit_cast(shortx4, p), __builtin_bit_cast(shortx4, m4), d, 0, 0, 0);
}
__device__ __forceinline__ floatx4 mixed(bf16x8 p, bf16x8 m, floatx4 d) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(p, m, d, 0, 0, 0);
}

struct TileArgs {
    const int32_t* group_first; const int32_t* group_count;
    int groups, group_tokens;                  // groups of this launch; NQ
    __bf16* e;                                 // [groups * NQ][ktiles][...]
    float* sums;                               // [groups * NQ][head_k][score_ranges]
    float* partial;                            // [groups * NQ][q_heads][value_ranges][value_dim]
    int ktiles, hp_log, head_k, kv_pad, page_log;
    int score_keys, score_ranges, value_keys, value_ranges;      // keys of a range (multiples of 32), ranges
};

// Where heads idx .. of key place i (0..15) of half s of a tile lie, from the tile's first element.
__device__ __forceinline__ int e_place(int head_k, int idx, int s, int i) {
    if (head_k == 16) return s * 256 + ((idx >> 2) * 16 + i) * 4 + (idx & 3);
    return ((idx >> 5) * 2 + s) * 512 + (((idx >> 3) & 3) * 16 + i) * 8 + (idx & 7);
}

// Which page a key lies in and its place there; page_log: log2(page_size), or -1 where that is no power of two.
struct PageOf {
    int page_size, page_log;
    __device__ __forceinline__ int block(int key) const { return page_log >= 0 ? key >> page_log : key / page_size; }
    __device__ __forceinline__ int place(int key) const { return page_log >= 0 ? key & (page_size - 1) : key % page_size; }
};

// One workgroup: a group's tokens x up to 16 RT rows (token, head of one kv head) x a range of keys; each of the four
// wavefronts takes every fourth tile of 32 keys.  Rows are the first operand (a lane ends up with four rows of one
// key: four heads of a token where a kv head has four), keys the second, straight from the pages: the next tile's rows
// are on their way while a tile's exponentials are taken, and the ids of the pages after that.
// HPL: log2 of the places a kv head's heads take, 2 for all from four on (a lane's four rows are then one token's).
template <int NKF, int RT, int HPL>
__global__ __launch_bounds__(256) void head_scores_kernel(HeadMixArgs a, TileArgs t) {
    constexpr int TOKENS = HPL == 0 ? 4 : HPL == 1 ? 2 : 1, PER = 4 / TOKENS;      // tokens of a lane's four rows; rows a token
    __shared__ float sum_lds[4][RT * 16];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, i16 = lane & 15, b = lane >> 4;
    const int g = (int)gridDim.x - 1 - (int)blockIdx.x;        // (a prompt's last groups have the most keys: first)
    const int kvh = blockIdx.y % t.kv_pad, row0 = (blockIdx.y / t.kv_pad) * RT * 16;
    const int first = t.group_first[g], count = t.group_count[g];
    const int hp_log = HPL < 2 ? HPL : t.hp_log, hp = 1 << hp_log, hg = a.q_heads / a.kv_heads, D = a.key_dim;
    const PageOf pages{a.page_size, t.page_log};
    const int p0 = a.positions[first], kend = p0 + count;
    const int32_t* table = a.block_table + (size_t)a.slots[first] * a.max_blocks;
    const bool real = kvh < a.kv_heads;
    const bool padded = !real || hg != hp;     // rows that stand for no head
    const bf16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
    bf16x8 qf[RT][NKF];
#pragma unroll
    for (int r = 0; r < RT; ++r) {
        const int row = row0 + r * 16 + i16, ti = row >> hp_log, hh = row & (hp - 1);
        const bool ok = real && ti < count && hh < hg;
        const __bf16* src = a.q + (size_t)(first + (ok ? ti : 0)) * a.q_stride + (size_t)(ok ? kvh * hg + hh : 0) * D;
#pragma unroll
        for (int kf = 0; kf < NKF; ++kf) {
            const int d = kf * 32 + b * 8;
            const bf16x8 v = *reinterpret_cast<const bf16x8*>(src + min(d, D - 8));
            qf[r][kf] = (ok && d < D) ? v : zero8;
        }
    }
    const int kt_step = t.score_keys / TK;
    const int kt_end = min((kend + TK - 1) / TK, ((int)blockIdx.z + 1) * kt_step);
    int kt = (int)blockIdx.z * kt_step + wave;
    const int te = TK * t.head_k, half = t.head_k == 16 ? 256 : 512;       // elements of a tile, of its half (one step of heads)
    // where the lane's rows go (tokens beyond the group's have no scratch; padded heads store their zeros)
    __bf16* dst[RT][TOKENS];
    bool stored[RT][TOKENS];
#pragma unroll
    for (int r = 0; r < RT; ++r)
#pragma unroll
        for (int x = 0; x < TOKENS; ++x) {
            const int row = row0 + r * 16 + 4 * b + x * PER, ti = row >> hp_log;
            stored[r][x] = ti < count;
            dst[r][x] = t.e + (((size_t)g * t.group_tokens + ti) * t.ktiles + kt) * te +
                        e_place(t.head_k, kvh * hp + (row & (hp - 1)), 0, i16);
        }
    float sums[RT][4];
#pragma unroll
    for (int r = 0; r < RT; ++r)
#pragma unroll
        for (int x = 0; x < 4; ++x) sums[r][x] = 0.f;
    // exp(cap tanh(x scale / cap)) = 2^(c1 - 2 c1 / (1 + 2^(x k))), c1 = cap log2(e), k = 2 log2(e) scale / cap
    const float c1 = a.softcap * 1.4426950408889634f, c2 = -2.0f * c1, kx = 2.0f * 1.4426950408889634f * (a.scale / a.softcap);
    const __bf16* kbase = a.k_pages + (size_t)(real ? kvh : 0) * a.page_size * D;
    const size_t page_elems = (size_t)a.kv_heads * a.page_size * D;
    const int lane_key = 8 * (i16 >> 2) + (i16 & 3);           // of the tile's first half; + 4: of its second
    bf16x8 kreg[2][NKF];
    int page[2];
    auto ask = [&](int kt) {                   // (clamped: loads behind no branch)
#pragma unroll
        for (int s = 0; s < 2; ++s) page[s] = table[pages.block(min(kt * TK + lane_key + 4 * s, kend - 1))];
    };
    auto fetch = [&](int kt) {
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            const int key = min(kt * TK + lane_key + 4 * s, kend - 1);
            const __bf16* kr = kbase + (size_t)max(page[s], 0) * page_elems + (size_t)pages.place(key) * D;
#pragma unroll
            for (int kf = 0; kf < NKF; ++kf) {
                const int d = kf * 32 + b * 8;
                const bf16x8 v = *reinterpret_cast<const bf16x8*>(kr + min(d, D - 8));
                kreg[s][kf] = d < D ? v : zero8;
            }
        }
    };
    if (kt < kt_end) {
        ask(kt);
        fetch(kt);
        ask(kt + 4);
    }
    for (; kt < kt_end; kt += 4) {
        floatx4 sc[RT][2];
#pragma unroll
        for (int r = 0; r < RT; ++r)
#pragma unroll
            for (int s = 0; s < 2; ++s) {
                floatx4 x = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int kf = 0; kf < NKF; ++kf) x = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[r][kf], kreg[s][kf], x, 0, 0, 0);
                sc[r][s] = x;
            }
        fetch(kt + 4);
        ask(kt + 8);
        // (the same in every lane: a tile that every token sees whole, no rows that stand for nothing)
        const bool plain = !padded && kt * TK + TK - 1 <= p0;
#pragma unroll
        for (int r = 0; r < RT; ++r) {
            const int row = row0 + r * 16 + 4 * b;               // the lane's rows row .. row + 3
#pragma unroll
            for (int s = 0; s < 2; ++s) {
                float e[4];
#pragma unroll
                for (int x = 0; x < 4; ++x) {
                    const float z = __builtin_amdgcn_exp2f(kx * sc[r][s][x]);
                    e[x] = __builtin_amdgcn_exp2f(__builtin_fmaf(c2, __builtin_amdgcn_rcpf(1.0f + z), c1));
                }
                if (!plain) {
                    const int key = kt * TK + lane_key + 4 * s - p0;
#pragma unroll
                    for (int x = 0; x < 4; ++x) {
                        const bool seen = real && ((row + x) & (hp - 1)) < hg && key <= ((row + x) >> hp_log);
                        e[x] = __uint_as_float(__float_as_uint(e[x]) & (seen ? 0xffffffffu : 0u));
                    }
                }
                bf16x4 e4;
#pragma unroll
                for (int x = 0; x < 4; ++x) {
                    sums[r][x] += e[x];
                    e4[x] = (__bf16)e[x];
                }
#pragma unroll
                for (int x = 0; x < TOKENS; ++x) {
                    if (!stored[r][x]) continue;
                    if (PER == 4) *reinterpret_cast<bf16x4*>(dst[r][x] + s * half) = e4;
                    else if (PER == 2) *reinterpret_cast<bf16x2*>(dst[r][x] + s * half) = bf16x2{e4[(2 * x) & 3], e4[(2 * x + 1) & 3]};
                    else dst[r][x][s * half] = e4[x];
                }
            }
#pragma unroll
            for (int x = 0; x < TOKENS; ++x) dst[r][x] += 4 * te;
        }
    }
    // a row's sum: over its 16 lanes, then over the wavefronts
#pragma unroll
    for (int r = 0; r < RT; ++r)
#pragma unroll
        for (int x = 0; x < 4; ++x) {
            float v = sums[r][x];
#pragma unroll
            for (int off = 1; off < 16; off <<= 1) v += __shfl_xor(v, off, MLR_WAVE);
            if (i16 == 0) sum_lds[wave][r * 16 + 4 * b + x] = v;
        }
    __syncthreads();
    for (int r = tid; r < RT * 16; r += 256) {
        const int row = row0 + r, ti = row >> hp_log, hh = row & (hp - 1);
        if (ti < count)
            t.sums[(((size_t)g * t.group_tokens + ti) * t.head_k + kvh * hp + hh) * t.score_ranges + blockIdx.z] =
                (sum_lds[0][r] + sum_lds[1][r]) + (sum_lds[2][r] + sum_lds[3][r]);
    }
}

// One workgroup (eight wavefronts): a group's tokens x `kv_block` kv heads' query heads x a range of keys.  A turn takes
// UNITS (token, tile of 32 keys) pairs -- sixteen tokens and one tile, or one token and eight tiles:
//   the wavefronts deal the units out, take exp(s) from the scratch, multiply by 1 / sum (32-bit), mix the heads on the
//   matrix cores and leave the block's mixed weights in LDS, [kv head][unit][head][32 keys];
//   then wavefront w multiplies kv head w / vs's weights (columns (token, head)) with its share w % vs of the value
//   channels, whose transposed rows come straight from the pages.
// Two LDS buffers: one barrier a turn.  HK: 16, 32 (one step of the mixing product, its operands in registers) or 0
// (any multiple of 32: `mix` and the inverse sums in LDS).
template <int HK, int CT, int VT, int NQ>
__global__ __launch_bounds__(512) void head_mix_values_kernel(HeadMixArgs a, TileArgs t, int kv_block) {
    constexpr int UNITS = NQ == 16 ? 16 : 8, UPW = UNITS / 8, KSUB = NQ == 16 ? 1 : 8;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds_raw[];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, i16 = lane & 15, b = lane >> 4;
    const int g = (int)gridDim.x - 1 - (int)blockIdx.x, kv0 = blockIdx.y * kv_block;
    const int first = t.group_first[g], count = t.group_count[g];
    const int hp = 1 << t.hp_log, hg = a.q_heads / a.kv_heads, V = a.value_dim, PS = a.page_size, H = a.q_heads;
    const int p0 = a.positions[first], kend = p0 + count;
    const int32_t* table = a.block_table + (size_t)a.slots[first] * a.max_blocks;
    const int head_k = HK == 0 ? t.head_k : HK, steps = HK == 0 ? t.head_k / 32 : 1;
    const int vs = 8 / kv_block, gl = wave / vs, vpart = wave % vs, kvh = kv0 + gl;
    const int block_rows = UNITS * hp + 1;     // 64-byte rows of a kv head in a buffer (one more: other banks)
    __bf16* w_lds = reinterpret_cast<__bf16*>(lds_raw);
    const int buffer = kv_block * block_rows * TK;
    float* inv_lds = reinterpret_cast<float*>(w_lds + 2 * buffer);                   // [NQ][head_k]   (HK == 0)
    __bf16* mix_lds = reinterpret_cast<__bf16*>(inv_lds + (HK == 0 ? NQ * head_k : 0));   // [steps][2][64][8]  (HK == 0)

    // 1 / sum of token ti's head of padded index idx
    auto inverse = [&](int ti, int idx) {
        const int kv = idx >> t.hp_log, hh = idx & (hp - 1);
        if (kv >= a.kv_heads || hh >= hg || ti >= count) return 0.f;
        const float* src = t.sums + (((size_t)g * t.group_tokens + ti) * t.head_k + idx) * t.score_ranges;
        float sum = a.sink_kind ? expf(sink_term(a, kv * hg + hh)) : 0.f;
        for (int z = 0; z < t.score_ranges; ++z) sum += src[z];
        return sum > 0.f ? 1.0f / sum : 0.f;
    };
    // mix[output head of local index hl][source head of padded index idx]
    auto mix_of = [&](int hl, int idx) {
        const int kv = kv0 + (hl >> t.hp_log), hh = hl & (hp - 1), skv = idx >> t.hp_log, sh = idx & (hp - 1);
        const bool ok = hl < kv_block * hp && kv < a.kv_heads && hh < hg && skv < a.kv_heads && sh < hg;
        return ok ? a.mix[(size_t)(kv * hg + hh) * H + skv * hg + sh] : 0.f;
    };
    constexpr int PER = HK == 16 ? 4 : 8;      // heads of a lane in one step
    float inv[UPW][PER];
    bf16x8 mixf[2];
    if (HK != 0) {
#pragma unroll
        for (int u = 0; u < UPW; ++u)
#pragma unroll
            for (int j = 0; j < PER; ++j) inv[u][j] = inverse(NQ == 16 ? wave * UPW + u : 0, b * PER + j);
#pragma unroll
        for (int n = 0; n < 2; ++n)
#pragma unroll
            for (int j = 0; j < 8; ++j) mixf[n][j] = j < PER ? (__bf16)mix_of(n * 16 + i16, b * PER + j) : (__bf16)0.f;
    } else {
        for (int i = tid; i < NQ * head_k; i += 512) inv_lds[i] = inverse(i / head_k, i % head_k);
        for (int i = tid; i < steps * 2 * 64 * 8; i += 512) {
            const int j = i & 7, l = (i >> 3) & 63, n = (i >> 9) & 1, st = i >> 10;
            mix_lds[i] = (__bf16)mix_of(n * 16 + (l & 15), st * 32 + (l >> 4) * 8 + j);
        }
        __syncthreads();
    }
    floatx4 acc[CT][VT];
#pragma unroll
    for (int c = 0; c < CT; ++c)
#pragma unroll
        for (int v = 0; v < VT; ++v) acc[c][v] = floatx4{0.f, 0.f, 0.f, 0.f};
    const int kt_first = (int)blockIdx.z * (t.value_keys / TK);
    const int kt_end = min((kend + TK - 1) / TK, kt_first + t.value_keys / TK);
    const size_t te = (size_t)TK * head_k;
    const __bf16* e_group = t.e + (size_t)g * t.group_tokens * t.ktiles * te;
    const PageOf pages{PS, t.page_log};
    const __bf16* vbase = a.v_pages + (size_t)(kvh < a.kv_heads ? kvh : 0) * V * PS;
    const size_t page_elems = (size_t)a.kv_heads * V * PS;

    const bool pv = kvh < a.kv_heads;
    // this lane's eight keys of a tile lie in one page: its id, and the transposed rows from there
    auto page_of = [&](int kt) { return table[pages.block(min(kt * TK + 8 * b, (kend - 1) & ~7))]; };
    auto values = [&](int kt, int page, bf16x8 (&vf)[VT]) {
        const int key = kt * TK + 8 * b;
        const __bf16* vr = vbase + (size_t)max(page, 0) * page_elems + pages.place(min(key, (kend - 1) & ~7));
#pragma unroll
        for (int v = 0; v < VT; ++v) vf[v] = *reinterpret_cast<const bf16x8*>(vr + (size_t)min((vpart + vs * v) * 16 + i16, V - 1) * PS);
    };
    // (places behind the last key hold anything)
    auto cut = [&](int kt, bf16x8 (&vf)[VT]) {
        if (kt * TK + TK <= kend) return;
        const int left = kend - (kt * TK + 8 * b);
#pragma unroll
        for (int v = 0; v < VT; ++v)
#pragma unroll
            for (int j = 0; j < 8; ++j)
                if (j >= left) vf[v][j] = (__bf16)0.f;
    };
    // the scratch of this wavefront's units of a turn (one step of heads: on its way a turn ahead)
    constexpr int EW = HK == 16 ? 4 : 8;
    typedef __attribute__((__vector_size__(EW * sizeof(__bf16)))) __bf16 bf16xe;
    bf16xe ereg[UPW][2];
    auto exps = [&](int kt0) {
        if (HK == 0) return;
#pragma unroll
        for (int u = 0; u < UPW; ++u) {
            const int unit = wave * UPW + u, ti = NQ == 16 ? min(unit, count - 1) : 0, kt = min(NQ == 16 ? kt0 : kt0 + unit, kt_end - 1);
            const __bf16* src = e_group + ((size_t)ti * t.ktiles + kt) * te + lane * EW;
#pragma unroll
            for (int s = 0; s < 2; ++s) ereg[u][s] = *reinterpret_cast<const bf16xe*>(src + s * 64 * EW);
        }
    };
    if (kt_first < kt_end) exps(kt_first);
    int page = kt_first < kt_end ? page_of(kt_first) : 0;
    int turn = 0;
    for (int kt0 = kt_first; kt0 < kt_end; kt0 += KSUB, turn ^= 1) {
        __bf16* wb = w_lds + turn * buffer;
        bf16x8 vf[VT];
        values(kt0, page, vf);                 // (on their way while the heads are mixed)
        if (NQ == 16) page = page_of(kt0 + 1);
#pragma unroll
        for (int u = 0; u < UPW; ++u) {
            const int unit = wave * UPW + u, ti = NQ == 16 ? unit : 0, kt = NQ == 16 ? kt0 : kt0 + unit;
            if (ti >= count || kt >= kt_end) continue;           // (the same in every lane)
            floatx4 d[2][2];
#pragma unroll
            for (int n = 0; n < 2; ++n)
#pragma unroll
                for (int s = 0; s < 2; ++s) d[n][s] = floatx4{0.f, 0.f, 0.f, 0.f};
            for (int st = 0; st < steps; ++st) {
                float f[PER];
#pragma unroll
                for (int j = 0; j < PER; ++j) f[j] = HK == 0 ? inv_lds[ti * head_k + st * 32 + b * 8 + j] : inv[u][j];
#pragma unroll
                for (int s = 0; s < 2; ++s) {
                    bf16xe ev = ereg[u][s];
                    if (HK == 0) ev = *reinterpret_cast<const bf16xe*>(e_group + ((size_t)ti * t.ktiles + kt) * te + (st * 2 + s) * 512 + lane * EW);
                    bf16xe p;
#pragma unroll
                    for (int j = 0; j < PER; ++j) p[j] = (__bf16)((float)ev[j] * f[j]);
#pragma unroll
                    for (int n = 0; n < 2; ++n)
                        if (n * 16 < kv_block * hp) d[n][s] = mixed(p, HK == 0 ? *reinterpret_cast<const bf16x8*>(mix_lds + ((st * 2 + n) * 64 + lane) * 8) : mixf[n], d[n][s]);
                }
            }
            // lane: head i16 of the column tile, keys 8 b .. 8 b + 7
#pragma unroll
            for (int n = 0; n < 2; ++n) {
                const int hl = n * 16 + i16;
                if (hl < kv_block * hp) {
                    bf16x8 w8;
#pragma unroll
                    for (int j = 0; j < 8; ++j) w8[j] = (__bf16)d[n][j >> 2][j & 3];
                    const int row = (hl >> t.hp_log) * block_rows + unit * hp + (hl & (hp - 1));
                    *reinterpret_cast<bf16x8*>(wb + row * TK + 8 * b) = w8;
                }
            }
        }
        exps(kt0 + KSUB);
        __syncthreads();
        if (pv) {
#pragma unroll 1
            for (int sub = 0; sub < KSUB; ++sub) {
                const int kt = kt0 + sub;
                if (kt >= kt_end) break;
                if (NQ != 16) {
                    // (single tokens: the next tile's values on their way while this one's are multiplied)
                    page = page_of(kt + 1);
                }
                cut(kt, vf);
                const __bf16* wr = wb + (gl * block_rows + (NQ == 16 ? 0 : sub * hp)) * TK + 8 * b;
#pragma unroll
                for (int c = 0; c < CT; ++c) {
                    const int col = c * 16 + i16;
                    // (columns beyond the heads of a single token repeat its last: their sums are dropped)
                    const bf16x8 wf = *reinterpret_cast<const bf16x8*>(wr + (NQ == 16 ? col : min(col, hp - 1)) * TK);
#pragma unroll
                    for (int v = 0; v < VT; ++v)
                        if ((vpart + vs * v) * 16 < V) acc[c][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[v], wf, acc[c][v], 0, 0, 0);
                }
                if (NQ != 16 && sub + 1 < KSUB) values(kt + 1, page, vf);
            }
        }
    }
    if (kvh >= a.kv_heads) return;
#pragma unroll
    for (int c = 0; c < CT; ++c) {
        const int col = c * 16 + i16, ti = NQ == 16 ? col >> t.hp_log : 0, hh = NQ == 16 ? col & (hp - 1) : col;
        if (ti >= count || hh >= hg) continue;
        float* dst = t.partial + ((((size_t)g * t.group_tokens + ti) * H + kvh * hg + hh) * t.value_ranges + blockIdx.z) * V;
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            const int ch = (vpart + vs * v) * 16 + 4 * b;
            if (ch < V) *reinterpret_cast<float4*>(dst + ch) = make_float4(acc[c][v][0], acc[c][v][1], acc[c][v][2], acc[c][v][3]);
        }
    }
}

// The ranges' shares added in ascending order, turned back, gated: a workgroup takes 256 channel pairs of a token of a
// group.
__global__ __launch_bounds__(256) void head_mix_finish_kernel(HeadMixArgs a, TileArgs t) {
    const int g = blockIdx.x, ti = blockIdx.y, V = a.value_dim, half = V >> 1;
    if (ti >= t.group_count[g]) return;
    const int m = t.group_first[g] + ti;
    const float* base = t.partial + ((size_t)g * t.group_tokens + ti) * a.q_heads * t.value_ranges * V;
    const int used = min(t.value_ranges, (a.positions[m] + t.value_keys) / t.value_keys);      // ranges that hold a key
    const float* cs = a.v_rope ? a.v_rope + (size_t)a.positions[m] * V : nullptr;
    const int o = blockIdx.z * 256 + threadIdx.x;
    if (o < a.q_heads * half) {
        const int h = o / half, j = o % half;
        const int c0 = a.v_interleaved ? 2 * j : j, c1 = a.v_interleaved ? 2 * j + 1 : j + half;
        float u = 0.f, v = 0.f;
        for (int z = 0; z < used; ++z) {
            const float* src = base + ((size_t)h * t.value_ranges + z) * V;
            u += src[c0];
            v += src[c1];
        }
        if (cs != nullptr) {
            const float co = cs[j], si = -cs[half + j];
            const float x = turn_x(u, v, co, si);
            v = turn_y(u, v, co, si);
            u = x;
        }
        if (a.gate != nullptr) {
            const float f = 1.0f / (1.0f + expf(-to_float(a.gate[(size_t)m * a.gate_stride + h])));
            u *= f;
            v *= f;
        }
        __bf16* dst = a.out + (size_t)m * a.out_stride + (size_t)h * V;
        dst[c0] = (__bf16)u;
        dst[c1] = (__bf16)v;
    }
}

template <int HK, int CT, int VT, int NQ>
static int launch_mix(const HeadMixArgs& a, const TileArgs& t, int kv_block, hipStream_t stream) {
    const int hp = 1 << t.hp_log, units = NQ == 16 ? 16 : 8;
    const size_t lds = (size_t)2 * kv_block * (units * hp + 1) * TK * sizeof(__bf16) +
                       (HK == 0 ? (size_t)NQ * t.head_k * sizeof(float) + (size_t)(t.head_k / 32) * 1024 * sizeof(__bf16) : 0);
    if (lds > 160 * 1024) return -4;
    static size_t raised = 48 * 1024;
    if (lds > raised) {
        if (hipFuncSetAttribute(reinterpret_cast<const void*>(&head_mix_values_kernel<HK, CT, VT, NQ>),
                                hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
            return -3;
        raised = lds;
    }
    head_mix_values_kernel<HK, CT, VT, NQ><<<dim3(t.groups, (a.kv_heads + kv_block - 1) / kv_block, t.value_ranges), 512, lds,
                                            stream>>>(a, t, kv_block);
    return (int)hipGetLastError();
}

template <int CT, int VT, int NQ>
static int launch_mix_heads(const HeadMixArgs& a, const TileArgs& t, int kv_block, hipStream_t stream) {
    if (t.head_k == 16) return launch_mix<16, CT, VT, NQ>(a, t, kv_block, stream);
    if (t.head_k == 32) return launch_mix<32, CT, VT, NQ>(a, t, kv_block, stream);
    return launch_mix<0, CT, VT, NQ>(a, t, kv_block, stream);
}

template <int NKF>
static int launch_scores(const HeadMixArgs& a, const TileArgs& t, hipStream_t stream) {
    const int rows = t.group_tokens << t.hp_log, tiles = (rows + 15) / 16;
    const int rt = tiles >= 4 ? 4 : tiles >= 2 ? 2 : 1;
    const dim3 grid(t.groups, t.kv_pad * ((tiles + rt - 1) / rt), t.score_ranges);
    if (grid.y > 65535 || grid.z > 65535) return -2;
    if (t.hp_log == 0) head_scores_kernel<NKF, 1, 0><<<grid, 256, 0, stream>>>(a, t);
    else if (t.hp_log == 1 && rt == 1) head_scores_kernel<NKF, 1, 1><<<grid, 256, 0, stream>>>(a, t);
    else if (t.hp_log == 1) head_scores_kernel<NKF, 2, 1><<<grid, 256, 0, stream>>>(a, t);
    else if (rt == 4) head_scores_kernel<NKF, 4, 2><<<grid, 256, 0, stream>>>(a, t);
    else if (rt == 2) head_scores_kernel<NKF, 2, 2><<<grid, 256, 0, stream>>>(a, t);
    else head_scores_kernel<NKF, 1, 2><<<grid, 256, 0, stream>>>(a, t);
    return (int)hipGetLastError();
}
#endif

extern "C" {

// out[m, h] for `rows` tokens, one workgroup each.  The heads' tiles and the output's sums live in LDS: -4 when they
// do not fit.
int mlr_head_mix_attention(const void* q, long q_stride, const void* k_pages, const void* v_pages, const int32_t* block_table,
                           int max_blocks, const int32_t* slots, const int32_t* positions, const float* mix,
                           const float* sink, float sink_value, int sink_kind, const float* v_rope, int v_interleaved,
                           const void* gate, long gate_stride, void* out, long out_stride, int rows, int q_heads,
                           int kv_heads, int key_dim, int value_dim, int page_size, float scale, float softcap,
                           hipStream_t stream) {
    if (rows <= 0) return 0;
    if (kv_heads <= 0 || q_heads % kv_heads != 0 || (v_rope && value_dim % 2 != 0) || sink_kind < 0 || sink_kind > 2 ||
        (sink_kind == 2 && sink == nullptr))
        return -1;
    const size_t lds = ((size_t)2 * q_heads * TILE_KEYS + (size_t)q_heads * value_dim + 2 * q_heads) * sizeof(float);
    if (lds > 150 * 1024) return -4;
    static size_t raised = 48 * 1024;
    if (lds > raised) {
        if (hipFuncSetAttribute(reinterpret_cast<const void*>(&head_mix_attention_kernel),
                                hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
            return -3;
        raised = lds;
    }
    HeadMixArgs a{(const elem_t*)q, q_stride, (const elem_t*)k_pages, (const elem_t*)v_pages, block_table, slots, positions,
                  mix, sink, sink_value, sink_kind, v_rope, v_interleaved, (const elem_t*)gate, gate_stride, (elem_t*)out,
                  out_stride, max_blocks, q_heads, kv_heads, key_dim, value_dim, page_size, scale, softcap};
    head_mix_attention_kernel<<<rows, 256, lds, stream>>>(a);
    return (int)hipGetLastError();
}

// The matrix-core form over `groups` groups of up to `group_tokens` (16 or 1) consecutive tokens of a request each.
// Scratch: e (bfloat16) groups * group_tokens * ktiles * 32 * head_k, sums (float) groups * group_tokens * head_k *
// score_ranges, partial (float) groups * group_tokens * q_heads * value_ranges * value_dim; ktiles: tiles of 32 keys
// that hold the longest context.  Ranges of score_keys / value_keys keys (multiples of 32; of 256 for single tokens'
// values) that together hold it too.  kv_block: kv heads of a workgroup of the second launch, 1, 2, 4 or 8.
// Returns 1 when the sizes are not this form's.
int mlr_head_mix_tiles(const void* q, long q_stride, const void* k_pages, const void* v_pages, const int32_t* block_table,
                       int max_blocks, const int32_t* slots, const int32_t* positions, const float* mix, const float* sink,
                       float sink_value, int sink_kind, const float* v_rope, int v_interleaved, const void* gate,
                       long gate_stride, void* out, long out_stride, const int32_t* group_first,
                       const int32_t* group_count, int groups, int group_tokens, int q_heads, int kv_heads, int key_dim,
                       int value_dim, int page_size, float scale, float softcap, void* e, float* sums, float* partial,
                       int ktiles, int head_pad, int head_k, int score_keys, int score_ranges, int value_keys,
                       int value_ranges, int kv_block, hipStream_t stream) {
#if MLR_BF16
    if (groups <= 0) return 0;
    int hp_log = 0;
    while ((1 << hp_log) < head_pad) ++hp_log;
    const int hg = kv_heads > 0 ? q_heads / kv_heads : 0;
    if (kv_heads <= 0 || q_heads % kv_heads != 0 || (1 << hp_log) != head_pad || hg > head_pad || head_pad > 32) return -1;
    if (key_dim % 8 != 0 || key_dim > 256 || value_dim % 16 != 0 || page_size % 8 != 0 || q_stride % 8 != 0 ||
        !(softcap > 0.f && softcap <= 60.f))
        return 1;
    if ((group_tokens != 16 && group_tokens != 1) || (head_k != 16 && head_k % 32 != 0) || head_k > 128 ||
        head_k % head_pad != 0 || head_k < kv_heads * head_pad || sink_kind < 0 || sink_kind > 2 ||
        (sink_kind == 2 && sink == nullptr))
        return -1;
    if (score_keys % TK != 0 || value_keys % (group_tokens == 1 ? 8 * TK : TK) != 0 || score_ranges < 1 || value_ranges < 1 ||
        score_keys <= 0 || value_keys <= 0 || (long)score_keys * score_ranges < (long)ktiles * TK ||
        (long)value_keys * value_ranges < (long)ktiles * TK || value_ranges > 65535)
        return -1;
    if ((kv_block != 1 && kv_block != 2 && kv_block != 4 && kv_block != 8) || kv_block * head_pad > 32) return -1;
    HeadMixArgs a{(const elem_t*)q, q_stride, (const elem_t*)k_pages, (const elem_t*)v_pages, block_table, slots, positions,
                  mix, sink, sink_value, sink_kind, v_rope, v_interleaved, (const elem_t*)gate, gate_stride, (elem_t*)out,
                  out_stride, max_blocks, q_heads, kv_heads, key_dim, value_dim, page_size, scale, softcap};
    int page_log = 0;
    while ((1 << page_log) < page_size) ++page_log;
    if ((1 << page_log) != page_size) page_log = -1;
    TileArgs t{group_first, group_count, groups, group_tokens, (__bf16*)e, sums, partial, ktiles, hp_log, head_k,
               head_k / head_pad, page_log, score_keys, score_ranges, value_keys, value_ranges};
    const int ct = group_tokens == 16 ? head_pad : (head_pad + 15) / 16;
    const int vt = (value_dim / 16 + 8 / kv_block - 1) / (8 / kv_block);
    if (ct * vt > 32 || vt > 8) return 1;
    const int nkf = (key_dim + 31) / 32;
    int rc = nkf <= 2 ? launch_scores<2>(a, t, stream) : nkf <= 4 ? launch_scores<4>(a, t, stream) : launch_scores<8>(a, t, stream);
    if (rc != 0) return rc;
    rc = 1;
#define MLR_MIX_CLASS(NQ, CT, VT)                                                     \
    if (rc == 1 && group_tokens == NQ && ct == CT && vt <= VT) rc = launch_mix_heads<CT, VT, NQ>(a, t, kv_block, stream);
    MLR_MIX_CLASS(16, 1, 2) MLR_MIX_CLASS(16, 1, 4) MLR_MIX_CLASS(16, 1, 8)
    MLR_MIX_CLASS(16, 2, 2) MLR_MIX_CLASS(16, 2, 4) MLR_MIX_CLASS(16, 2, 8)
    MLR_MIX_CLASS(16, 4, 1) MLR_MIX_CLASS(16, 4, 2) MLR_MIX_CLASS(16, 4, 4)
    MLR_MIX_CLASS(16, 8, 2) MLR_MIX_CLASS(16, 8, 4) MLR_MIX_CLASS(16, 16, 2) MLR_MIX_CLASS(16, 32, 1)
    MLR_MIX_CLASS(1, 1, 1) MLR_MIX_CLASS(1, 1, 2) MLR_MIX_CLASS(1, 1, 4) MLR_MIX_CLASS(1, 1, 8) MLR_MIX_CLASS(1, 2, 2) MLR_MIX_CLASS(1, 2, 8)
#undef MLR_MIX_CLASS
    if (rc != 0) return rc;
    head_mix_finish_kernel<<<dim3(groups, group_tokens, (q_heads * (value_dim / 2) + 255) / 256), 256, 0, stream>>>(a, t);
    return (int)hipGetLastError();
#else
    return 1;
#endif
}

}  // extern "C"
