// Causal attention on the matrix cores for bfloat16 rows, in three forms:
//   shared    every query row looks at the same key rows, whose first columns are also the values (attention in
//             latent space: the key rows are the cache itself);
//   rows      the queries of a group of heads look at the rows of their key/value head, [value | key] (grouped attention);
//   expanded  keys and values of every head were formed beforehand: a key is [own part | part shared by all heads],
//             values come transposed ([value column][key]).
//
// A wave owns 16 (or 2 x 16) query rows.  It forms the scores transposed, S^T = K Q^T (v_mfma_f32_16x16x32_bf16 with
// the keys as rows), so that lane l holds scores of query l % 16 only: keys 16 t + 4 (l / 16) + i.  These registers
// are, without any exchange, the B operand of O^T = V^T P^T if lane group l / 16 takes the keys
// {4 g + i, 16 + 4 g + i} of a 32-key step as its eight k places; V^T is read from LDS in that order.  Running maximum
// and sum are one value per lane.  Scores, softmax and sums are fp32.
//
// A tile of keys is copied global -> LDS by direct 16-byte loads.  Key rows: chunk c of row r at place c ^ (r & 7).
// Query columns beyond the real width are zero, so whatever finite values sit there in the key rows do not count.
#include "dense_common.h"

namespace a81w41 {
namespace {

typedef __attribute__((ext_vector_type(4))) short s16x4;
typedef __attribute__((ext_vector_type(8))) short s16x8;
typedef __attribute__((address_space(3))) s16x4* lds_s16x4;
constexpr float kLog2e = 1.4426950408889634f;
constexpr float kLowest = -1e30f;

// DK, DV: capacities for all and for value columns of a tile row; the scores take its columns from KEY0 on (rows form: the
// key part, 0 otherwise).  KT keys per tile, NBUF tiles in LDS.
// COLS (few rows): all four waves take the same query rows; each scores its 16 keys of a tile, the scores meet in LDS,
// and each sums its quarter of the value columns.
template <int DK, int DV, int KEY0, int WAVES, int QS, int KT, int NBUF, bool EXPANDED, bool COLS>
__global__ __launch_bounds__(64 * WAVES, 1) void attend_kernel(AttendArgs<bf16> a) {
    constexpr int CK = DK / 8;                    // 16-byte chunks of a key row
    constexpr int kKeyBytes = KT * DK * 2, kValueBytes = EXPANDED ? DV * KT * 2 : 0;
    constexpr int CV = KT / 8;                    // chunks of a value row (transposed)
    constexpr int kBuf = kKeyBytes + kValueBytes;
    constexpr int KS = (DK - KEY0) / 32, VF = DV / 16 / (COLS ? WAVES : 1), kRows = 16 * QS * (COLS ? 1 : WAVES);
    static_assert(DK % 64 == 0 && KEY0 % 32 == 0 && DV % (COLS ? 16 * WAVES : 16) == 0 && KT % 32 == 0 && (!EXPANDED || CV == 8), "tile sizes");
    constexpr int kScoreRow = 16 * QS + 4;  // floats of a key's scores in LDS: lane groups fall into different banks
    static_assert(!COLS || KT == 16 * WAVES, "a wave scores 16 keys of a tile");
    __shared__ __attribute__((aligned(128))) uint8_t lds[NBUF * kBuf];
    __shared__ float scores[COLS ? KT * kScoreRow : 1];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l15 = lane & 15, g = lane >> 4;
    const int row_wave = COLS ? 0 : wave, f0 = COLS ? wave * VF : 0;  // first 16 value columns of this wave
    const int z = blockIdx.y;
    // the longest rows first
    const int row0 = ((int)gridDim.x - 1 - (int)blockIdx.x) * kRows;
    const int pos = min(max(a.pos_dev[0], 0), a.max_seq - 1);
    const int last_row = min(row0 + kRows, a.rows) - 1;
    const int wg_keys = min(pos + last_row / a.rows_per_token, a.max_seq - 1) + 1;  // keys any row of the workgroup sees
    auto chunk_begin = [&](int key) { return a.chunk ? key - key % a.chunk : 0; };
    int key_begin = chunk_begin(min(pos + row0 / a.rows_per_token, a.max_seq - 1)), key_end = wg_keys;
    if (a.splits > 1) {
        const int from = chunk_begin(pos), all = min(pos + (a.rows - 1) / a.rows_per_token, a.max_seq - 1) + 1 - from;
        const int share = ((all + a.splits - 1) / a.splits + KT - 1) / KT * KT, begin = from + (int)blockIdx.z * share;
        key_end = min(begin + share, wg_keys);
        key_begin = min(max(begin, key_begin), key_end);
    }
    const bf16* k_own = a.k_own + z * a.k_own_head;
    const bf16* v_t = EXPANDED ? a.v_t + (size_t)z * a.dv * a.ld_v : nullptr;
    const int own_chunks = a.k_own_width >> 3, all_chunks = own_chunks + (EXPANDED ? a.k_shared_width >> 3 : 0);
    auto copy_tile = [&](int key0, int buf) {
        uint8_t* base = lds + buf * kBuf;
        for (int n = wave; n < KT * CK / 64; n += WAVES) {
            const int q = n * 64 + lane, r = q / CK, c = (q % CK) ^ (r & 7);
            const size_t key = min(key0 + r, wg_keys - 1);
            const bf16* src = k_own + key * a.ld_k_own;
            if constexpr (KEY0 > 0) {
                if (c < KEY0 / 8)
                    src += c < (a.v_width >> 3) ? c * 8 : 0;
                else if (c - KEY0 / 8 < own_chunks)
                    src += a.v_width + (c - KEY0 / 8) * 8;
            } else if (c < own_chunks)
                src += c * 8;
            else if (EXPANDED && c < all_chunks)
                src = a.k_shared + key * a.ld_k_shared + (c - own_chunks) * 8;
            copy16_to_lds(src, base + n * 1024);
        }
        if constexpr (EXPANDED)
            for (int n = wave; n < DV * CV / 64; n += WAVES) {
                const int q = n * 64 + lane, r = q >> 3, c = (q & 7) ^ (r & 7);
                copy16_to_lds(v_t + (size_t)min(r, a.dv - 1) * a.ld_v + key0 + c * 8, base + kKeyBytes + n * 1024);
            }
    };
    // query operands
    bf16x8 qf[QS][KS];
    int limit[QS], first[QS];  // last and first visible key of this lane's query
#pragma unroll
    for (int s = 0; s < QS; s++) {
        const int r = row0 + (row_wave * QS + s) * 16 + l15, rc = min(r, a.rows - 1);
        const int token = rc / a.rows_per_token, last = min(pos + token, a.max_seq - 1);
        limit[s] = r < a.rows ? last : -1;
        first[s] = chunk_begin(last);
        const bf16* src = a.q + z * a.q_head + (size_t)token * a.q_token + (rc - token * a.rows_per_token) * a.ld_q;
#pragma unroll
        for (int k = 0; k < KS; k++) {
            uint4 u = make_uint4(0, 0, 0, 0);
            const int c = k * 4 + g;
            if (c < all_chunks) u = *reinterpret_cast<const uint4*>(src + c * 8);
            qf[s][k] = *reinterpret_cast<const bf16x8*>(&u);
        }
    }
    f32x4 acc[QS][VF];
    float mx[QS], sum[QS];
#pragma unroll
    for (int s = 0; s < QS; s++) {
        const bool sink = a.sink && (a.splits == 1 || blockIdx.z == 0);  // one lane group of one share counts it
        mx[s] = sink ? 0.f : kLowest;
        sum[s] = sink && g == 0 ? 1.f : 0.f;
#pragma unroll
        for (int f = 0; f < VF; f++) acc[s][f] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    // Values that are columns of the key rows come by transposing reads (ds_read_b64_tr_b16): in a group of 16 lanes lane
    // i names four columns of key 4 g + i / 4 and receives its own column of the four keys.  The exclusive or of the chunk
    // places touches the low three bits of 2 f + ..., so four offsets serve all f.
    int value_at[4];
    if constexpr (!EXPANDED) {
#pragma unroll
        for (int f = 0; f < 4; f++) {
            const int r = 4 * g + (l15 >> 2);
            value_at[f] = r * (DK * 2) + (((2 * (f0 + f) + ((l15 >> 1) & 1)) ^ (r & 7)) << 4) + (l15 & 1) * 8;
        }
    }
    const float scale = a.scale * kLog2e;
    const int n_tiles = (key_end - key_begin + KT - 1) / KT;
    if (NBUF > 1 && n_tiles > 0) copy_tile(key_begin, 0);
    for (int tile = 0; tile < n_tiles; tile++) {
        const int key0 = key_begin + tile * KT;
        if (NBUF == 1) {
            if (tile) __syncthreads();  // nobody still reads the tile
            copy_tile(key0, 0);
        }
        __builtin_amdgcn_s_waitcnt(0x0070);
        __syncthreads();
        if (NBUF > 1 && tile + 1 < n_tiles) copy_tile(key0 + KT, (tile + 1) % NBUF);
        const uint8_t* kb = lds + (tile % NBUF) * kBuf;
        const uint8_t* vb = kb + kKeyBytes;
        f32x4 sc[QS][KT / 16];
        auto score = [&](int t) {
#pragma unroll
            for (int s = 0; s < QS; s++) sc[s][t] = f32x4{0.f, 0.f, 0.f, 0.f};
            const uint8_t* row = kb + ((COLS ? wave : t) * 16 + l15) * (DK * 2);
#pragma unroll
            for (int k = 0; k < KS; k++) {
                const bf16x8 kf = *reinterpret_cast<const bf16x8*>(row + (((KEY0 / 8 + k * 4 + g) ^ (l15 & 7)) << 4));
#pragma unroll
                for (int s = 0; s < QS; s++) sc[s][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[s][k], sc[s][t], 0, 0, 0);
            }
        };
        if constexpr (COLS) {
            score(0);
#pragma unroll
            for (int s = 0; s < QS; s++)
#pragma unroll
                for (int i = 0; i < 4; i++) scores[(wave * 16 + 4 * g + i) * kScoreRow + s * 16 + l15] = sc[s][0][i];
            dense_lds_barrier();
#pragma unroll
            for (int s = 0; s < QS; s++)
#pragma unroll
                for (int t = 0; t < KT / 16; t++)
#pragma unroll
                    for (int i = 0; i < 4; i++) sc[s][t][i] = scores[(t * 16 + 4 * g + i) * kScoreRow + s * 16 + l15];
        } else {
#pragma unroll
            for (int t = 0; t < KT / 16; t++) score(t);
        }
        bf16x8 pf[QS][KT / 32];
#pragma unroll
        for (int s = 0; s < QS; s++) {
            float m = mx[s];
#pragma unroll
            for (int t = 0; t < KT / 16; t++)
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    const int key = key0 + t * 16 + 4 * g + i;
                    const float v = sc[s][t][i] * scale;
                    sc[s][t][i] = key <= limit[s] && key >= first[s] && key < key_end ? v : kLowest;
                    m = fmaxf(m, sc[s][t][i]);
                }
            m = fmaxf(m, __shfl_xor(m, 16, 64));
            m = fmaxf(m, __shfl_xor(m, 32, 64));
            const float keep = exp2f(mx[s] - m);
            float add = 0.f;
#pragma unroll
            for (int t = 0; t < KT / 16; t++)
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    const float p = sc[s][t][i] > kLowest ? exp2f(sc[s][t][i] - m) : 0.f;
                    add += p;
                    pf[s][t >> 1][(t & 1) * 4 + i] = (bf16)p;
                }
            sum[s] = sum[s] * keep + add;
            mx[s] = m;
            if (__any(keep != 1.f)) {
#pragma unroll
                for (int f = 0; f < VF; f++) acc[s][f] *= keep;
            }
        }
#pragma unroll
        for (int u = 0; u < KT / 32; u++)
#pragma unroll
            for (int f = 0; f < VF; f++) {
                bf16x8 vf;
                if constexpr (EXPANDED) {
                    const int r = (f0 + f) * 16 + l15;
                    const uint8_t* row = vb + r * (KT * 2);
                    const int c0 = u * 4 + (g >> 1);
                    uint2 lo = *reinterpret_cast<const uint2*>(row + ((c0 ^ (r & 7)) << 4) + (g & 1) * 8);
                    uint2 hi = *reinterpret_cast<const uint2*>(row + (((c0 + 2) ^ (r & 7)) << 4) + (g & 1) * 8);
                    const uint4 w = make_uint4(lo.x, lo.y, hi.x, hi.y);
                    vf = *reinterpret_cast<const bf16x8*>(&w);
                } else {
                    const uint8_t* at = kb + value_at[f & 3] + (f >> 2) * 128 + u * 32 * (DK * 2);
                    const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4)(at));
                    const s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4)(at + 16 * (DK * 2)));
                    const s16x8 both = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
                    vf = *reinterpret_cast<const bf16x8*>(&both);
                }
#pragma unroll
                for (int s = 0; s < QS; s++) acc[s][f] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[s][u], acc[s][f], 0, 0, 0);
            }
    }
    // lane l holds value columns 16 f + 4 g + i of query l % 16
#pragma unroll
    for (int s = 0; s < QS; s++) {
        float all = sum[s];
        all += __shfl_xor(all, 16, 64);
        all += __shfl_xor(all, 32, 64);
        const int r = row0 + (row_wave * QS + s) * 16 + l15;
        if (r >= a.rows) continue;
        if (a.splits > 1) {
            const size_t at = ((size_t)blockIdx.z * gridDim.y + z) * a.rows + r;
            if (g == 0 && f0 == 0) {
                a.part_stats[2 * at] = mx[s];
                a.part_stats[2 * at + 1] = all;
            }
            float* dst = a.part + at * a.ld_part;
#pragma unroll
            for (int f = 0; f < VF; f++)
                if ((f0 + f) * 16 + 4 * g < a.ld_part) *reinterpret_cast<f32x4*>(dst + (f0 + f) * 16 + 4 * g) = acc[s][f];
        } else {
            float inv = 1.0f / all;
            if (a.head_gate) inv *= sigmoid(a.head_gate[(size_t)r * a.ld_gate + z]);
            const int token = r / a.rows_per_token;
            bf16* dst = a.out + z * a.out_head + (size_t)token * a.out_token + (r - token * a.rows_per_token) * a.ld_out;
#pragma unroll
            for (int f = 0; f < VF; f++)
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    const int d = (f0 + f) * 16 + 4 * g + i;
                    if (d < a.dv) dst[d] = (bf16)(acc[s][f][i] * inv);
                }
        }
    }
}

// out row = sum_s w_s part_s / sum_s w_s sum_s with w_s = 2^(m_s - max m); one workgroup per head's row and 256 columns
__global__ __launch_bounds__(256) void merge_shares_kernel(AttendArgs<bf16> a, int heads) {
    __shared__ float w[kAttendMaxSplits];
    __shared__ float norm;
    const int all_rows = heads * a.rows, at = blockIdx.x, t = threadIdx.x;
    if (t < 64) {
        float m = t < a.splits ? a.part_stats[2 * ((size_t)t * all_rows + at)] : kLowest;
        const float l = t < a.splits ? a.part_stats[2 * ((size_t)t * all_rows + at) + 1] : 0.f;
        const float top = dense_wave_max(m);
        const float mine = exp2f(m - top);
        if (t < a.splits) w[t] = mine;
        const float total = dense_wave_sum(t < a.splits ? mine * l : 0.f);
        if (t == 0) norm = 1.0f / total;
    }
    __syncthreads();
    const int d = blockIdx.y * 256 + t;
    if (d >= a.dv) return;
    float s = 0.f;
    for (int k = 0; k < a.splits; k++) s = fmaf(w[k], a.part[((size_t)k * all_rows + at) * a.ld_part + d], s);
    const int z = at / a.rows, r = at - z * a.rows, token = r / a.rows_per_token;
    a.out[z * a.out_head + (size_t)token * a.out_token + (r - token * a.rows_per_token) * a.ld_out + d] = (bf16)(s * norm);
}
static_assert(kAttendMaxSplits <= 64, "the merge reads one share per lane");

template <int DK, int DV, int KEY0, int WAVES, int QS, int KT, int NBUF, bool EXPANDED, bool COLS>
hipError_t launch_kernel(const AttendArgs<bf16>& a, int heads, hipStream_t s) {
    constexpr int rows = 16 * QS * (COLS ? 1 : WAVES);
    hipLaunchKernelGGL((attend_kernel<DK, DV, KEY0, WAVES, QS, KT, NBUF, EXPANDED, COLS>), dim3((a.rows + rows - 1) / rows, heads, a.splits),
                       dim3(64 * WAVES), 0, s, a);
    return hipGetLastError();
}
template <int DK, int DV>
hipError_t launch_shared(const AttendArgs<bf16>& a, hipStream_t s) {
    return a.rows <= kAttendFewRows ? launch_kernel<DK, DV, 0, 4, 1, 64, 2, false, true>(a, 1, s)
                                    : launch_kernel<DK, DV, 0, 4, 1, 32, 1, false, false>(a, 1, s);
}
// key and value columns: D at most each
template <int D, int QS>
hipError_t launch_rows(const AttendArgs<bf16>& a, int heads, hipStream_t s) {
    return a.rows <= kAttendFewRows ? launch_kernel<2 * D, D, D, 4, 1, 64, 2, false, true>(a, heads, s)
                                    : launch_kernel<2 * D, D, D, 4, QS, 64, 2, false, false>(a, heads, s);
}
template <int DK, int DV>
hipError_t launch_expanded(const AttendArgs<bf16>& a, int heads, hipStream_t s) {
    return launch_kernel<DK, DV, 0, 4, 2, 64, 2, true, false>(a, heads, s);
}

}  // namespace

bool attend_shared_fits(int dk, int dv) { return dk <= 576 && dv <= 512; }
bool attend_rows_fits(int key, int value) { return key % 8 == 0 && value % 8 == 0 && key <= 256 && value <= 256; }
bool attend_expanded_fits(int own, int shared, int dv) { return own % 8 == 0 && shared % 8 == 0 && own + shared <= 320 && dv <= 256; }

hipError_t launch_attend_shared(const AttendArgs<bf16>& a, hipStream_t s) {
    const int dk = a.k_own_width;
    if (dk <= 192 && a.dv <= 128) return launch_shared<192, 128>(a, s);
    if (dk <= 320 && a.dv <= 256) return launch_shared<320, 256>(a, s);
    return launch_shared<576, 512>(a, s);
}

hipError_t launch_attend_rows(const AttendArgs<bf16>& a, int heads, hipStream_t s) {
    const int widest = a.k_own_width > a.v_width ? a.k_own_width : a.v_width;
    if (widest <= 64) return launch_rows<64, 2>(a, heads, s);
    if (widest <= 128) return launch_rows<128, 2>(a, heads, s);
    return launch_rows<256, 1>(a, heads, s);
}

hipError_t launch_attend_expanded(const AttendArgs<bf16>& a, int heads, hipStream_t s) {
    const int dk = a.k_own_width + a.k_shared_width;
    if (dk <= 128 && a.dv <= 64) return launch_expanded<128, 64>(a, heads, s);
    if (dk <= 192 && a.dv <= 128) return launch_expanded<192, 128>(a, heads, s);
    return launch_expanded<320, 256>(a, heads, s);
}

hipError_t launch_merge_shares(const AttendArgs<bf16>& a, int heads, hipStream_t s) {
    hipLaunchKernelGGL(merge_shares_kernel, dim3(heads * a.rows, (a.dv + 255) / 256), dim3(256), 0, s, a, heads);
    return hipGetLastError();
}

}  // namespace a81w41
