// JSON and safetensors readers (see checkpoint.hpp); host code only.
#include "checkpoint.hpp"

#include <cmath>
#include <cstdlib>
#include <cstring>
#include <fcntl.h>
#include <fstream>
#include <sstream>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

namespace litenn_hip
{
	namespace
	{
		struct Parser
		{
			const char* p;
			const char* end;
			const std::string& what;
			int depth = 0;

			[[noreturn]] void bad(const char* why) const { throw std::runtime_error(what + ": " + why); }

			void space()
			{
				while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r'))
				{
					++p;
				}
			}

			bool take(char c)
			{
				space();
				if (p < end && *p == c)
				{
					++p;
					return true;
				}
				return false;
			}

			void word(const char* w)
			{
				const size_t n = strlen(w);
				if (static_cast<size_t>(end - p) < n || memcmp(p, w, n) != 0)
				{
					bad("malformed JSON");
				}
				p += n;
			}

			unsigned hex4()
			{
				unsigned v = 0;
				for (int i = 0; i < 4; ++i, ++p)
				{
					if (p >= end)
					{
						bad("unterminated JSON string");
					}
					const char c = *p;
					const int d = c >= '0' && c <= '9' ? c - '0' : (c | 32) >= 'a' && (c | 32) <= 'f' ? (c | 32) - 'a' + 10 : -1;
					if (d < 0)
					{
						bad("malformed JSON escape");
					}
					v = v * 16 + static_cast<unsigned>(d);
				}
				return v;
			}

			void utf8(std::string& s, unsigned c)
			{
				const auto put = [&](unsigned b) { s.push_back(static_cast<char>(b)); };
				if (c < 0x80)
				{
					put(c);
				}
				else if (c < 0x800)
				{
					put(0xc0 | (c >> 6));
					put(0x80 | (c & 63));
				}
				else if (c < 0x10000)
				{
					put(0xe0 | (c >> 12));
					put(0x80 | ((c >> 6) & 63));
					put(0x80 | (c & 63));
				}
				else
				{
					put(0xf0 | (c >> 18));
					put(0x80 | ((c >> 12) & 63));
					put(0x80 | ((c >> 6) & 63));
					put(0x80 | (c & 63));
				}
			}

			std::string text()
			{
				std::string s;
				while (true)
				{
					if (p >= end)
					{
						bad("unterminated JSON string");
					}
					char c = *p++;
					if (c == '"')
					{
						return s;
					}
					if (c != '\\')
					{
						s.push_back(c);
						continue;
					}
					if (p >= end)
					{
						bad("unterminated JSON string");
					}
					c = *p++;
					switch (c)
					{
					case 'n': s.push_back('\n'); break;
					case 't': s.push_back('\t'); break;
					case 'r': s.push_back('\r'); break;
					case 'b': s.push_back('\b'); break;
					case 'f': s.push_back('\f'); break;
					case 'u':
					{
						unsigned u = hex4();
						if (u >= 0xd800 && u < 0xdc00 && end - p >= 2 && p[0] == '\\' && p[1] == 'u')
						{
							p += 2;
							u = 0x10000 + ((u - 0xd800) << 10) + ((hex4() - 0xdc00) & 0x3ff);
						}
						utf8(s, u);
						break;
					}
					case '"':
					case '\\':
					case '/': s.push_back(c); break;
					default: bad("malformed JSON escape");
					}
				}
			}

			Json value()
			{
				if (++depth > 64)
				{
					bad("JSON nested too deeply");
				}
				space();
				if (p >= end)
				{
					bad("unexpected end of JSON");
				}
				Json v;
				switch (*p)
				{
				case '{':
					++p;
					v.kind = Json::Object;
					if (!take('}'))
					{
						do
						{
							if (!take('"'))
							{
								bad("malformed JSON object");
							}
							std::string key = text();
							if (!take(':'))
							{
								bad("malformed JSON object");
							}
							v.members.emplace_back(std::move(key), value());
						} while (take(','));
						if (!take('}'))
						{
							bad("malformed JSON object");
						}
					}
					break;
				case '[':
					++p;
					v.kind = Json::Array;
					if (!take(']'))
					{
						do
						{
							v.items.push_back(value());
						} while (take(','));
						if (!take(']'))
						{
							bad("malformed JSON array");
						}
					}
					break;
				case '"':
					++p;
					v.kind = Json::String;
					v.text = text();
					break;
				case 't':
					word("true");
					v.kind = Json::Bool;
					v.boolean = true;
					break;
				case 'f':
					word("false");
					v.kind = Json::Bool;
					break;
				case 'n': word("null"); break;
				default:
				{
					const char* q = p;
					while (q < end && (strchr("+-.eE", *q) || (*q >= '0' && *q <= '9')))
					{
						++q;
					}
					const std::string digits(p, q);
					char* stop = nullptr;
					v.kind = Json::Number;
					v.number = strtod(digits.c_str(), &stop);
					if (digits.empty() || *stop != 0)
					{
						bad("malformed JSON number");
					}
					p = q;
				}
				}
				--depth;
				return v;
			}
		};
	} // namespace

	Json Json::parse(const char* begin, size_t size, const std::string& what)
	{
		Parser parser{ begin, begin + size, what };
		Json v = parser.value();
		parser.space();
		if (parser.p != parser.end)
		{
			parser.bad("text after the JSON value");
		}
		return v;
	}

	const Json* Json::find(const std::string& key) const
	{
		for (const auto& m : members)
		{
			if (m.first == key)
			{
				return &m.second;
			}
		}
		return nullptr;
	}

	const Json& Json::at(const std::string& key) const
	{
		const Json* v = find(key);
		if (!v)
		{
			throw std::runtime_error("configuration has no '" + key + "'");
		}
		return *v;
	}

	double Json::real(const std::string& key) const
	{
		const Json& v = at(key);
		if (v.kind != Number || !std::isfinite(v.number))
		{
			throw std::runtime_error("configuration: '" + key + "' is not a number");
		}
		return v.number;
	}

	int Json::integer(const std::string& key, int low, int high) const
	{
		const double v = real(key);
		if (v != std::floor(v) || v < low || v > high)
		{
			throw std::runtime_error("configuration: '" + key + "' is not a whole number in [" + std::to_string(low) + ", " +
			                         std::to_string(high) + "]");
		}
		return static_cast<int>(v);
	}

	const std::string& Json::string(const std::string& key) const
	{
		const Json& v = at(key);
		if (v.kind != String)
		{
			throw std::runtime_error("configuration: '" + key + "' is not a string");
		}
		return v.text;
	}

	std::string read_text_file(const std::string& path)
	{
		std::ifstream f(path, std::ios::binary);
		if (!f)
		{
			throw std::runtime_error("cannot open '" + path + "'");
		}
		std::ostringstream s;
		s << f.rdbuf();
		return s.str();
	}

	Safetensors::Safetensors(const std::string& path)
	{
		const int fd = open(path.c_str(), O_RDONLY | O_CLOEXEC);
		if (fd < 0)
		{
			throw std::runtime_error("cannot open '" + path + "'");
		}
		struct stat st{};
		if (fstat(fd, &st) == 0 && st.st_size > 8)
		{
			size_ = static_cast<size_t>(st.st_size);
			map_ = mmap(nullptr, size_, PROT_READ, MAP_PRIVATE, fd, 0);
			if (map_ == MAP_FAILED)
			{
				map_ = nullptr;
			}
		}
		close(fd);
		if (!map_)
		{
			throw std::runtime_error("cannot map '" + path + "'");
		}
		try
		{
			const uint8_t* base = static_cast<const uint8_t*>(map_);
			uint64_t header = 0;
			for (int i = 7; i >= 0; --i)
			{
				header = (header << 8) | base[i];
			}
			if (header > size_ - 8)
			{
				throw std::runtime_error(path + ": header longer than the file");
			}
			const size_t data_at = 8 + static_cast<size_t>(header), data_size = size_ - data_at;
			const Json root = Json::parse(reinterpret_cast<const char*>(base) + 8, static_cast<size_t>(header), path);
			for (const auto& m : root.members)
			{
				if (m.first == "__metadata__")
				{
					continue;
				}
				CheckpointTensor t;
				t.dtype = m.second.string("dtype");
				size_t count = 1;
				for (const Json& d : m.second.at("shape").items)
				{
					if (d.kind != Json::Number || d.number < 0 || d.number > 1e12 || d.number != std::floor(d.number))
					{
						throw std::runtime_error(path + ": bad shape of '" + m.first + "'");
					}
					t.shape.push_back(static_cast<size_t>(d.number));
					if (t.shape.back() && count > size_ / t.shape.back())
					{
						throw std::runtime_error(path + ": bad shape of '" + m.first + "'");
					}
					count *= t.shape.back();
				}
				const Json& off = m.second.at("data_offsets");
				if (off.items.size() != 2 || off.items[0].kind != Json::Number || off.items[1].kind != Json::Number ||
				    !(off.items[0].number >= 0) || !(off.items[1].number >= off.items[0].number) ||
				    off.items[1].number > static_cast<double>(data_size))
				{
					throw std::runtime_error(path + ": '" + m.first + "' lies outside the file");
				}
				const size_t from = static_cast<size_t>(off.items[0].number), to = static_cast<size_t>(off.items[1].number);
				t.data = base + data_at + from;
				t.bytes = to - from;
				const size_t width = t.dtype == "BF16" || t.dtype == "F16" ? 2 : t.dtype == "F32" || t.dtype == "I32" ? 4 : 0;
				if (width && count * width != t.bytes)
				{
					throw std::runtime_error(path + ": '" + m.first + "' has another size than its shape");
				}
				tensors_.emplace(m.first, std::move(t));
			}
		}
		catch (...)
		{
			munmap(map_, size_);
			throw;
		}
	}

	Safetensors::~Safetensors()
	{
		if (map_)
		{
			munmap(map_, size_);
		}
	}
} // namespace litenn_hip
